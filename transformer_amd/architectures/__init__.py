"""Registry entries. Importing the package registers them."""
from . import kunitar, linonex, llama, luduvik, saredra, vametar, zirutar  # noqa: F401
