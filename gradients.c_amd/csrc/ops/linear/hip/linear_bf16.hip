/* The few-row projection kernels over BF16 operands: linear.hip compiled with the other element type (linear_elem.h). */
#define GD_LINEAR_BF16 1
#include "linear.hip"
