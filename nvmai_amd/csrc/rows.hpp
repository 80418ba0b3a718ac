// Which sequence and position each row of a call is, and the angle of a position: shared by the kernels of the dense
// models.  gfx950.
#pragma once

#include "common.hpp"

namespace nvmai {

// Where a row's token sits: by arrays (a decode batch) or consecutive from (slot, position) (a prompt's portion).
struct SeqRows {
    const uint32_t *slots, *positions;
    uint32_t slot, position;
    __device__ __forceinline__ uint32_t slot_of(uint32_t r) const { return slots ? slots[r] : slot; }
    __device__ __forceinline__ uint32_t position_of(uint32_t r) const { return positions ? positions[r] : position + r; }
};

// (cos, sin) of position * inv_freq with the angle reduced in double: exact to fp32 at any position.
__device__ __forceinline__ void position_angle(uint32_t position, double inv_freq, float& c, float& s) {
    double a = (double)position * inv_freq;
    a -= 6.283185307179586476925 * rint(a * 0.15915494309189533577);
    sincosf((float)a, &s, &c);
}

// The first position of a sliding window that ends at `position`; window 0 reaches back to the start.
__device__ __forceinline__ uint32_t first_key(uint32_t position, uint32_t window) {
    return window != 0u && position + 1u > window ? position + 1u - window : 0u;
}

}  // namespace nvmai
