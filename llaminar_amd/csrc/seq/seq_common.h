// Shared by the sequence-model kernels: operand types of the matrix unit, tiled weights,
// reductions, launch-time checks.
//
// Every kernel is a template over the operand type T: bf16 (16-bit matrix operands, 32-bit sums)
// or float (true 32-bit products on v_mfma_f32_16x16x4_f32).  One "k-step" is 32 elements of the
// inner dimension in both: lane (r = lane & 15, g = lane >> 4) holds elements 8 g .. 8 g + 7 of
// row (or column) r.  For float the step is eight 16x16x4 products, product j pairing element
// 8 g + j of both operands, so the two operand layouts are the same.  A 16x16 result leaves lane
// (c, g) with rows 4 g .. 4 g + 3 of column c.
#pragma once

#include <hip/hip_runtime.h>

#include <cstdint>

#include "ql_host.h"

namespace llamql
{
    constexpr int WAVE64 = 64;
    constexpr int PAD = 64; // every inner dimension is padded with zeros to a multiple of this

    typedef __bf16 bf16;
    typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
    typedef bf16 bf16x8 __attribute__((ext_vector_type(8)));
    typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
    typedef float f32x4 __attribute__((ext_vector_type(4)));
    typedef float f32x8 __attribute__((ext_vector_type(8)));

    template <typename T>
    struct Operand;

    template <>
    struct Operand<bf16>
    {
        using V = bf16x8;
        // bf16 pieces that carry a 32-bit value exactly (8 + 8 + 8 significant bits)
        static constexpr int PIECES = 3;
        static __device__ __forceinline__ f32x4 mma(V a, V b, f32x4 c)
        {
            return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
        }
        static __device__ __forceinline__ V from_weights(u32x4 raw) { return __builtin_bit_cast(bf16x8, raw); }
        static __device__ __forceinline__ V load(const bf16 *p) { return *reinterpret_cast<const bf16x8 *>(p); }
    };

    template <>
    struct Operand<float>
    {
        using V = f32x8;
        static constexpr int PIECES = 1;
        static __device__ __forceinline__ f32x4 mma(V a, V b, f32x4 c)
        {
#pragma unroll
            for (int j = 0; j < 8; ++j)
                c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
            return c;
        }
        static __device__ __forceinline__ V from_weights(u32x4 raw)
        {
            return __builtin_convertvector(__builtin_bit_cast(bf16x8, raw), f32x8);
        }
        static __device__ __forceinline__ V load(const float *p)
        {
            const f32x4 a = *reinterpret_cast<const f32x4 *>(p), b = *reinterpret_cast<const f32x4 *>(p + 4);
            return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
        }
    };

    // 32-bit values as matrix operands.  bf16: the value minus what earlier pieces already carry,
    // piece after piece, so a product over all pieces is that of the 32-bit value; float: itself.
    template <typename T, int N>
    __device__ __forceinline__ void split_pieces(f32x8 x, typename Operand<T>::V (&out)[N])
    {
        if constexpr (sizeof(T) == 4)
            out[0] = x;
        else
        {
#pragma unroll
            for (int p = 0; p < N; ++p)
            {
                out[p] = __builtin_convertvector(x, bf16x8);
                if (p + 1 < N)
                    x -= __builtin_convertvector(out[p], f32x8);
            }
        }
    }

    template <typename T>
    __device__ __forceinline__ float rounded(float x)
    {
        return (float)(T)x;
    }

    // Tiled weights: a matrix of N rows (padded to 16) and K columns (padded to PAD) is stored as
    // [N/16][K/32][64 lanes][8] bf16: the 16-byte piece of lane (r, g) of a k-step, so a wavefront
    // reads a 16-row k-step as one contiguous kilobyte.
    __device__ __forceinline__ const u32x4 *weight_tile(const void *w, size_t tile, int ksteps, int lane)
    {
        return static_cast<const u32x4 *>(w) + tile * (size_t)ksteps * 64 + lane;
    }

    __device__ __forceinline__ float wave_sum64(float v)
    {
#pragma unroll
        for (int off = 32; off > 0; off >>= 1)
            v += __shfl_xor(v, off, WAVE64);
        return v;
    }

    // sum over the workgroup, the same value in every thread; s holds one float per wavefront
    template <int THREADS>
    __device__ __forceinline__ float block_sum(float v, float *s)
    {
        v = wave_sum64(v);
        __syncthreads();
        if ((threadIdx.x & 63) == 0)
            s[threadIdx.x >> 6] = v;
        __syncthreads();
        float t = 0.0f;
#pragma unroll
        for (int w = 0; w < THREADS / 64; ++w)
            t += s[w];
        return t;
    }

    __device__ __forceinline__ float gelu_tanh(float z)
    {
        return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
    }
    __device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }

    // Largest logits of one token by one wavefront: ids and softmax weights over the chosen ones,
    // lane t < top holding the t-th.  A tie goes to the lower index.  n <= 64 * ROUTE_MAX.
    constexpr int ROUTE_MAX = 16; // up to 1024 experts
    __device__ __forceinline__ void route_wave(const float *z, int n, int top, int lane, int &id, float &weight)
    {
        if (n <= 64)
        {
            // an expert a lane: its place is the number of experts ahead of it
            const float v = lane < n ? z[lane] : -INFINITY;
            int place = 0;
            for (int e = 0; e < n; ++e)
            {
                const float o = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), e));
                place += o > v || (o == v && e < lane) ? 1 : 0;
            }
            id = 0;
            for (int t = 0; t < top; ++t)
            {
                const unsigned long long at = __ballot(place == t && lane < n);
                const int who = at ? __builtin_ctzll(at) : t; // (none: only with logits that are not numbers)
                if (lane == t)
                    id = who;
            }
            const float mine = __shfl(v, id, WAVE64), first = __shfl(v, __builtin_amdgcn_readfirstlane(id), WAVE64);
            const float e = lane < top ? expf(mine - first) : 0.0f;
            weight = e / wave_sum64(e);
            return;
        }
        float v[ROUTE_MAX];
#pragma unroll
        for (int i = 0; i < ROUTE_MAX; ++i)
        {
            const int e = i * 64 + lane;
            v[i] = i * 64 < n && e < n ? z[e] : -INFINITY;
        }
        id = 0;
        float mine = -INFINITY, first = 0.0f;
        for (int t = 0; t < top; ++t)
        {
            float best = -INFINITY;
            int bi = 0x7fffffff;
#pragma unroll
            for (int i = 0; i < ROUTE_MAX; ++i)
                if (i * 64 < n && v[i] > best)
                {
                    best = v[i];
                    bi = i * 64 + lane;
                }
#pragma unroll
            for (int off = 32; off > 0; off >>= 1)
            {
                const float ov = __shfl_xor(best, off, WAVE64);
                const int oi = __shfl_xor(bi, off, WAVE64);
                if (ov > best || (ov == best && oi < bi))
                {
                    best = ov;
                    bi = oi;
                }
            }
            if (bi >= n) // only with logits that are not numbers
                bi = t;
            if (t == 0)
                first = best;
            if (lane == t)
            {
                id = bi;
                mine = best;
            }
#pragma unroll
            for (int i = 0; i < ROUTE_MAX; ++i)
                if (i * 64 + lane == bi)
                    v[i] = -INFINITY;
        }
        const float e = lane < top ? expf(mine - first) : 0.0f;
        weight = e / wave_sum64(e);
    }

    // Operand whose inner index runs along the rows of a row-major LDS array: lane (r, g) gets
    // rows 8 g .. 8 g + 7 of column r.  base points at row 0, column 0 of the 32 x 16 block.
    // bf16 uses the transposing LDS read: sixteen lanes read a 4 x 16 block, lane i supplying the
    // address of row i / 4, columns 4 (i % 4) .. + 3, and lane i receives column i.
    __device__ __forceinline__ bf16x8 load_columns(const bf16 *base, int ld, int lane)
    {
        typedef __attribute__((address_space(3))) bf16x4 *lds4;
        const int i = lane & 15, g = lane >> 4;
        const bf16 *p = base + (8 * g + (i >> 2)) * ld + (i & 3) * 4;
        const bf16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)p);
        const bf16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds4)(p + 4 * ld));
        return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
    }
    __device__ __forceinline__ f32x8 load_columns(const float *base, int ld, int lane)
    {
        const float *p = base + 8 * (lane >> 4) * ld + (lane & 15);
        f32x8 v;
#pragma unroll
        for (int j = 0; j < 8; ++j)
            v[j] = p[j * ld];
        return v;
    }

    inline int ceil_div(int a, int b) { return (a + b - 1) / b; }
    inline int round_up(int a, int b) { return ceil_div(a, b) * b; }
} // namespace llamql
