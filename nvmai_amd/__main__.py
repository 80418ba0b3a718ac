"""Command line: python -m nvmai_amd {generate,replay} ..."""
import sys

from .cli import main

sys.exit(main())
