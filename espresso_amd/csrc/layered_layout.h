// Host-side layout helpers of layered runtimes: matrices are uploaded with their heads and widths padded.
#pragma once

#include <stdint.h>

#include <cstring>
#include <vector>

namespace esp {
namespace layered {

inline int up(int v, int to) { return (v + to - 1) / to * to; }

// Copies rows [first, first + count) of a host matrix [..][cols] to rows at.. of dst [..][ld].
inline void place_rows(const std::vector<uint16_t> &src, int cols, int first, int count, std::vector<uint16_t> *dst, int ld, int at, int at_col = 0) {
    for (int r = 0; r < count; r++)
        std::memcpy(dst->data() + (size_t)(at + r) * ld + at_col, src.data() + (size_t)(first + r) * cols, (size_t)cols * 2);
}

}  // namespace layered
}  // namespace esp
