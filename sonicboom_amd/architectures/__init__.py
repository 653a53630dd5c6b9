"""Built-in architectures; importing the package registers them."""
from . import dudatar, fitatar, nalasun, nidasun, qwen2, rasizen, tatelorn  # noqa: F401
