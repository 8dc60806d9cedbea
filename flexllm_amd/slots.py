"""Which sequence lives in which slot of a model (a slot holds one sequence's cached rows and states on the device)."""


class NoFreeSlot(RuntimeError):
    pass


class SlotPool:
    def __init__(self, n, reset):
        """reset(slot) starts a slot afresh; it is called when the slot is handed out."""
        self._free = list(range(n - 1, -1, -1))
        self._of = {}
        self._reset = reset

    def acquire(self, key):
        """Slot of a new sequence `key`, started afresh."""
        if key in self._of:
            raise KeyError("%r already has a slot" % (key,))
        if not self._free:
            raise NoFreeSlot("all %d slots hold a sequence" % len(self._of))
        slot = self._free.pop()
        self._of[key] = slot
        self._reset(slot)
        return slot

    def slot(self, key):
        """Slot of `key`, handed out on first use."""
        return self._of[key] if key in self._of else self.acquire(key)

    def release(self, key):
        self._free.append(self._of.pop(key))

    def __contains__(self, key):
        return key in self._of

    @property
    def free(self):
        return len(self._free)
