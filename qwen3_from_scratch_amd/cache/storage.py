"""The device memory behind the cache manager's page numbers and slots."""

from dataclasses import dataclass, field

import torch


@dataclass
class LayerCacheView:
    """What one mixer sees of the cache in one step."""

    paged: dict = field(default_factory=dict)   # name of a PagedTensor -> (pages, *page shape)
    block_table: torch.Tensor = None            # int32 (B, W), this step's requests in batch order
    writes: bool = True
    state: torch.Tensor = None                  # (slots, *state_shape); index with batch.state_slots
    runs: dict = field(default_factory=dict)    # name of a tensor per run of tokens -> (pages, *page shape)
    run_table: torch.Tensor = None              # int32 (B, W): the pages of each request's runs


class CacheStorage:
    """Per paged group, one tensor for each `PagedTensor` its mixers declared: (planes, pages,
    *page shape) in the declared dtype or the activation dtype; the in-page layout is the
    mixer's own (see `PagedTensor`), this class only allocates what is declared. Per state
    group one tensor (planes, slots, *shape), zeroed per slot at admission. Every group has one
    page, and every state group one slot, more than the manager hands out (`spare_page`,
    `spare_slot`): rows that only fill a batch up to a size a captured graph exists for write
    there."""

    def __init__(self, manager, act_dtype, device):
        self.manager = manager
        self.device = torch.device(device)
        self.paged = []                                # per group {name: tensor}
        for grp in manager.groups:
            tensors = {}
            for t in grp.tensors:
                shape = (len(grp.planes), grp.pool.num_pages + 1) + t.page_shape(manager.page_size)
                tensors[t.name] = torch.zeros(shape, dtype=t.dtype or act_dtype, device=self.device)
            self.paged.append(tensors)
        self.states = []
        for grp in manager.state_groups:
            self.states.append(torch.zeros(
                (len(grp.planes), manager.max_requests + 1) + tuple(grp.shape),
                dtype=grp.dtype, device=self.device))
        self._block_tables = None

    def spare_page(self, group):
        return self.manager.groups[group].pool.num_pages

    @property
    def spare_slot(self):
        return self.manager.max_requests

    def bytes(self):
        tensors = [t for group in self.paged for t in group.values()] + self.states
        return sum(t.numel() * t.element_size() for t in tensors)

    def clear_fresh_slots(self):
        fresh, self.manager.fresh_slots = self.manager.fresh_slots, []
        if fresh and self.states:
            index = torch.tensor(fresh, dtype=torch.long, device=self.device)
            for t in self.states:
                t[:, index] = 0

    def keep_states(self, slots):
        """Copies of the states in `slots` (a device tensor of slot numbers), to be put back by
        `put_states`: a step that is run for another reason than its result (the eager run before a
        graph is captured) must leave no trace in states that the real step then continues. Pages
        need no such care: the real step writes the same keys to the same places again."""
        index = slots.long()
        return index, [t.index_select(1, index) for t in self.states]

    def put_states(self, kept):
        index, copies = kept
        for t, copy in zip(self.states, copies):
            t.index_copy_(1, index, copy)

    def bind(self, block_tables):
        """`block_tables`: per paged group the step's int32 (B, W) device tensor."""
        self._block_tables = block_tables

    def view(self, plane, writes=True):
        m = self.manager
        view = LayerCacheView(writes=writes)
        g = m.group_of_plane[plane]
        if g >= 0:
            local = m.groups[g].planes.index(plane)
            view.paged = {name: tensor[local] for name, tensor in self.paged[g].items()}
            view.block_table = self._block_tables[g]
        r = m.run_group_of_plane[plane]
        if r >= 0:
            local = m.groups[r].planes.index(plane)
            view.runs = {name: tensor[local] for name, tensor in self.paged[r].items()}
            view.run_table = self._block_tables[r]
        s = m.state_group_of_plane[plane]
        if s >= 0:
            local = m.state_groups[s].planes.index(plane)
            view.state = self.states[s][local]
        return view
