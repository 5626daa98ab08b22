/* 256 x 256 tiles over [K,N] weights of the many-row F16 projection kernel (linear_tile.hip). */
#define GD_LINEAR_TILE_PART 2
#include "linear_tile.hip"
