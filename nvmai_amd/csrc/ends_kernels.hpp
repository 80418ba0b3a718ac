// The two ends of a dense model: embedding rows, the cap of the logits, argmax.  gfx950, wave64.
#pragma once

#include "rows.hpp"

namespace nvmai {

// Rows of a BF16 table as 32-bit residual rows; an id past the table gives zeros.  scale: factor of the table's rows;
// inv_freq (nullptr: none): plus the sinusoid of the row's position, entry 2 i its sine and 2 i + 1 its cosine at
// inv_freq[i]; act (nullptr: none): the row once more as activations.
struct EmbedParams {
    const uint16_t* table;
    const uint32_t* ids;
    float* out;
    void* act;
    const double* inv_freq;
    SeqRows rows;
    uint32_t table_stride, out_stride, act_stride, d, vocab;
    float scale;
};

template <int ACT>
__global__ __launch_bounds__(256) void embed_rows_kernel(EmbedParams p) {
    const uint32_t row = blockIdx.y, pair = blockIdx.x * 256u + threadIdx.x, j = 2u * pair;
    if (j >= p.d) return;
    const uint32_t id = p.ids[row];
    const bool two = j + 1u < p.d;
    const uint16_t* e = p.table + (size_t)id * p.table_stride + j;
    float a = 0.0f, b = 0.0f;
    if (id < p.vocab) {
        a = bf16_to_f32(e[0]) * p.scale;
        b = two ? bf16_to_f32(e[1]) * p.scale : 0.0f;
    }
    if (p.inv_freq) {
        float c, s;
        position_angle(p.rows.position_of(row), p.inv_freq[pair], c, s);
        a += s;
        b += c;
    }
    float* out = p.out + (size_t)row * p.out_stride + j;
    out[0] = a;
    if (two) out[1] = b;
    if (p.act) {
        act_t<ACT>* h = static_cast<act_t<ACT>*>(p.act) + (size_t)row * p.act_stride + j;
        h[0] = f32_to_act<ACT>(a);
        if (two) h[1] = f32_to_act<ACT>(b);
    }
}

// x <- cap tanh(x / cap)
__global__ __launch_bounds__(256) void softcap_rows_kernel(float* x, uint32_t x_stride, uint32_t n, float cap) {
    const uint32_t j = blockIdx.x * 256u + threadIdx.x;
    if (j >= n) return;
    float* v = x + (size_t)blockIdx.y * x_stride + j;
    *v = cap * tanhf(*v / cap);
}

// Index of the largest finite value of each row, ties to the lower index, 0 when none is finite.  A candidate is one
// 64-bit key: the value in the upper half (mapped so that unsigned order is the order of the floats), the complement
// of the index in the lower; 0 = none.
constexpr uint32_t ARGMAX_BLOCKS = 64;

__device__ __forceinline__ uint64_t argmax_key(float v, uint32_t index) {
    const uint32_t b = __float_as_uint(v);
    if ((b & 0x7F800000u) == 0x7F800000u) return 0ull;         // infinite or not a number
    const uint32_t o = b == 0x80000000u ? 0x80000000u : (b & 0x80000000u) ? ~b : b | 0x80000000u;    // -0 ranks as 0
    return ((uint64_t)o << 32) | (uint32_t)~index;
}

__device__ __forceinline__ uint64_t argmax_block(uint64_t best, uint64_t* lds) {
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) {
        const uint64_t o = ((uint64_t)shfl_xor_u((uint32_t)(best >> 32), off) << 32) | shfl_xor_u((uint32_t)best, off);
        best = o > best ? o : best;
    }
    if ((threadIdx.x & 63u) == 0) lds[threadIdx.x >> 6] = best;
    __syncthreads();
    for (int w = 0; w < 4; ++w) best = lds[w] > best ? lds[w] : best;
    return best;
}

__global__ __launch_bounds__(256) void argmax_stage1_kernel(const float* x, uint32_t x_stride, uint32_t n, uint64_t* part) {
    __shared__ uint64_t lds[4];
    const float* row = x + (size_t)blockIdx.y * x_stride;
    uint64_t best = 0;
#pragma unroll 4
    for (uint32_t j = blockIdx.x * 256u + threadIdx.x; j < n; j += 256u * gridDim.x) {
        const uint64_t k = argmax_key(row[j], j);
        best = k > best ? k : best;
    }
    best = argmax_block(best, lds);
    if (threadIdx.x == 0) part[blockIdx.y * ARGMAX_BLOCKS + blockIdx.x] = best;
}

__global__ __launch_bounds__(256) void argmax_stage2_kernel(const uint64_t* part, uint32_t blocks, uint32_t* out) {
    __shared__ uint64_t lds[4];
    const uint64_t best = argmax_block(threadIdx.x < blocks ? part[blockIdx.x * ARGMAX_BLOCKS + threadIdx.x] : 0ull, lds);
    if (threadIdx.x == 0) out[blockIdx.x] = best == 0ull ? 0u : ~(uint32_t)best;
}

}  // namespace nvmai
