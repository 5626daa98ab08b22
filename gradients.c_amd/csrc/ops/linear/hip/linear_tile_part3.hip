/* 128 x 128 and 192 x 256 tiles of the many-row F16 projection kernel (linear_tile.hip). */
#define GD_LINEAR_TILE_PART 3
#include "linear_tile.hip"
