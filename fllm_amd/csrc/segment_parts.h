// Long segments of a step cut into parts of PART tokens that run side by side.
//
// Where part `part` of the segment that begins at row seg_r0 keeps what it hands on: no two parts of a step share an index,
// and the largest is below rows / PART + segments.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

template <int PART> __host__ __device__ inline int part_index(int seg_r0, int seg, int part) { return seg_r0 / PART + seg + part; }

// The grid of a step in parts has one workgroup (times whatever else it spans) an index that a part may have: workgroup w finds
// the last segment whose first index is not above w (the first indices grow with the segment) and is that segment's part
// w - first index, if the segment has so many.
template <int PART> __device__ inline void find_part(int w, const int32_t *seg_start, int num_segs, int &seg, int &part) {
    int lo = 0, hi = num_segs - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (part_index<PART>(seg_start[mid], mid, 0) <= w) lo = mid;
        else hi = mid - 1;
    }
    seg = lo;
    part = w - part_index<PART>(seg_start[lo], lo, 0);
}
