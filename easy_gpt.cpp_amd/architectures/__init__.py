"""Built-in architectures; importing this package registers them."""
from . import bubetar, karesun, kezolix, nebanex, pekasun, qwen2, tipezen  # noqa: F401
