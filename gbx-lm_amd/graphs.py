"""Capturing launches in a HIP graph."""
from __future__ import annotations

import contextlib
import gc

import torch


@contextlib.contextmanager
def capture(graph, **kwargs):
    """``torch.cuda.graph`` with Python's cyclic garbage collector switched off while the capture runs.  A collection may fall between
    any two launches, and what it frees may include a graph of an earlier engine (an engine and its caches refer to each other, so
    they go by collection, not by reference count): destroying a graph synchronises the device, which a capture in progress forbids --
    the destructor's error then ends the process."""
    was = gc.isenabled()
    gc.disable()
    try:
        with torch.cuda.graph(graph, **kwargs):
            yield
    finally:
        if was:
            gc.enable()
