"""Importing this package registers the architectures the library ships (GPT-2, Salopel, Kodatar, Rotutar, Gavasun,
Loselix)."""

from . import gavasun, gpt2, kodatar, loselix, rotutar, salopel  # noqa: F401
