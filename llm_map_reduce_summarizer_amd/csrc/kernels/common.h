// Shared helpers for the gfx950 (CDNA4) kernels of mrsum.
//
// Conventions (all kernels):
//   * bf16 tensors are moved as 16-byte vectors (8 x bf16 per lane); scalar
//     bf16 traffic is never used on a hot path (cdna_hip_programming.md G13).
//   * math is fp32; fp32 -> bf16 is a plain cast, which hipcc lowers to
//     v_cvt_pk_bf16_f32 (RNE, NaN-preserving).
//   * wavefront = 64 lanes; every block size is a multiple of 64.
//   * every extern "C" launcher takes raw device pointers + a hipStream_t,
//     never allocates or synchronises (legal inside hipGraph capture) and
//     returns hipGetLastError() as an int.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <algorithm>
#include <math.h>

#define MRSUM_API extern "C" __attribute__((visibility("default")))

typedef __bf16 bf16;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef short short4v __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));  // 16-B staging register (SROA-friendly, unlike HIP's uint4 struct)

static constexpr int WAVE = 64;

__device__ __forceinline__ float bf16_bits_to_f32(uint32_t bits16) {
    return __uint_as_float(bits16 << 16);
}

// 8 packed bf16 (one uint4) -> 8 floats
__device__ __forceinline__ void unpack8(const uint4 v, float* f) {
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
    f[4] = __uint_as_float(v.z << 16); f[5] = __uint_as_float(v.z & 0xffff0000u);
    f[6] = __uint_as_float(v.w << 16); f[7] = __uint_as_float(v.w & 0xffff0000u);
}

__device__ __forceinline__ uint32_t pack2(float a, float b) {
    bf16 x = (bf16)a, y = (bf16)b;
    return (uint32_t)__builtin_bit_cast(uint16_t, x) | ((uint32_t)__builtin_bit_cast(uint16_t, y) << 16);
}

__device__ __forceinline__ uint4 pack8(const float* f) {
    return make_uint4(pack2(f[0], f[1]), pack2(f[2], f[3]), pack2(f[4], f[5]), pack2(f[6], f[7]));
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
    return v;
}

// Block-wide sum for blockDim.x <= 1024 (uses 16 floats of LDS).
__device__ __forceinline__ float block_sum(float v, float* red) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
    v = wave_sum(v);
    if (lane == 0) red[wid] = v;
    __syncthreads();
    float t = lane < nw ? red[lane] : 0.f;
    t = wave_sum(t);
    __syncthreads();
    return t;
}

// Loads that bypass this CU's L1 (buffer_load ... sc1, aux 16): they read the XCD's L2 / memory copy, so
// a split-K last arriver can read other workgroups' write-through (sc1) stores of THIS launch without an
// agent-scope acquire (buffer_inv sc1 + wait, ~1.7 us) -- the hand-off form of MI355X_MICROARCH.md
// "Valid forms" row 1 / cdna_hip_programming.md Guideline 16: every payload store sc1 and drained before
// the ticket add, the last adder loads after its add returned, the other waves after a barrier, EVERY
// load of the payload such a load.  ``base`` must be wave-uniform (one buffer resource), ``off`` bytes.
__device__ __forceinline__ __amdgpu_buffer_rsrc_t sc1_rsrc(const void* base) {
    return __builtin_amdgcn_make_buffer_rsrc(const_cast<void*>(base), (short)0, 0x7fffffff, 0x00020000);
}
__device__ __forceinline__ float4 ld_sc1_f4(__amdgpu_buffer_rsrc_t r, int off) {
    const u32x4 v = __builtin_amdgcn_raw_buffer_load_b128(r, off, 0, 16);
    return make_float4(__uint_as_float(v[0]), __uint_as_float(v[1]), __uint_as_float(v[2]), __uint_as_float(v[3]));
}
__device__ __forceinline__ float2 ld_sc1_f2(__amdgpu_buffer_rsrc_t r, int off) {
    typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
    const u32x2 v = __builtin_amdgcn_raw_buffer_load_b64(r, off, 0, 16);
    return make_float2(__uint_as_float(v[0]), __uint_as_float(v[1]));
}

// Gated linear unit of the gate_up GEMM epilogues: g sigmoid(alpha g) (u + shift) with g <= limit, |u| <= limit.
// The defaults are SwiGLU.
struct GluArgs {
    float limit = INFINITY, alpha = 1.f, shift = 0.f;
};
__device__ __forceinline__ float glu(float g, float u, const GluArgs& a) {
    g = fminf(g, a.limit);
    u = fminf(fmaxf(u, -a.limit), a.limit);
    return g / (1.f + __expf(-a.alpha * g)) * (u + a.shift);
}

// Attention output form: head h of row t goes to columns [h * pitch, (h + 1) * pitch) of the row, times
// gate[t * gate_ld + h] when a gate is given.
struct AttnEpi {
    const float* gate;
    int gate_ld;
    int pitch;
};

// A projection's result as its consumer kernels read it: fp32 split-K slabs [S][rows][ld] to be summed (PARTS,
// S >= 1), or 16-bit rows [rows][ld].
struct ProjSrc {
    const void* p;
    int S;
    size_t slab;  // elements between slabs
    int ld;
};

template <bool PARTS>
__device__ __forceinline__ float proj_at(const ProjSrc& s, int row, int col) {
    const size_t i = (size_t)row * s.ld + col;
    if constexpr (!PARTS) return (float)reinterpret_cast<const bf16*>(s.p)[i];
    const float* f = reinterpret_cast<const float*>(s.p) + i;
    float a = 0.f;
#pragma unroll 4
    for (int k = 0; k < s.S; ++k) a += f[k * s.slab];
    return a;
}

// 8 (4) consecutive columns; col and ld are multiples of 8 (4)
template <bool PARTS>
__device__ __forceinline__ void proj8(const ProjSrc& s, int row, int col, float* o) {
    const size_t i = (size_t)row * s.ld + col;
    if constexpr (!PARTS) {
        unpack8(*reinterpret_cast<const uint4*>(reinterpret_cast<const bf16*>(s.p) + i), o);
    } else {
        const float* f = reinterpret_cast<const float*>(s.p) + i;
#pragma unroll
        for (int j = 0; j < 8; ++j) o[j] = 0.f;
#pragma unroll 4
        for (int k = 0; k < s.S; ++k) {
            const float4 a = *reinterpret_cast<const float4*>(f + k * s.slab);
            const float4 b = *reinterpret_cast<const float4*>(f + k * s.slab + 4);
            o[0] += a.x; o[1] += a.y; o[2] += a.z; o[3] += a.w;
            o[4] += b.x; o[5] += b.y; o[6] += b.z; o[7] += b.w;
        }
    }
}

template <bool PARTS>
__device__ __forceinline__ float4 proj4(const ProjSrc& s, int row, int col) {
    const size_t i = (size_t)row * s.ld + col;
    if constexpr (!PARTS) {
        const uint2 v = *reinterpret_cast<const uint2*>(reinterpret_cast<const bf16*>(s.p) + i);
        return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u),
                           __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u));
    } else {
        const float* f = reinterpret_cast<const float*>(s.p) + i;
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
        for (int k = 0; k < s.S; ++k) {
            const float4 a = *reinterpret_cast<const float4*>(f + k * s.slab);
            o.x += a.x; o.y += a.y; o.z += a.z; o.w += a.w;
        }
        return o;
    }
}

// A batch as segments, one per sequence: segment i covers rows [cu[i], cu[i + 1]) (cu null: row i) and continues state
// slot slots[i] at absolute position pos0[i].
struct SegArgs {
    const int* cu;       // [n + 1] or null (one row per segment)
    const int* row_seg;  // [T] segment of every row (cu given)
    const int* slots;
    const int* pos0;
};

__device__ __forceinline__ void load8(const float* p, float* f) {
    const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}

__device__ __forceinline__ void ld8(const float* p, float* f) { load8(p, f); }
__device__ __forceinline__ void ld8(const bf16* p, float* f) { unpack8(*reinterpret_cast<const uint4*>(p), f); }

// 8 / 4 values to bf16 or fp32 storage (aligned)
__device__ __forceinline__ void store8(bf16* p, const float* f) { *reinterpret_cast<uint4*>(p) = pack8(f); }
__device__ __forceinline__ void store8(float* p, const float* f) {
    reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
    reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
}
__device__ __forceinline__ void store4(bf16* p, const float4& f) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack2(f.x, f.y), pack2(f.z, f.w));
}
__device__ __forceinline__ void store4(float* p, const float4& f) { *reinterpret_cast<float4*>(p) = f; }

__device__ __forceinline__ float logistic(float x) { return 1.f / (1.f + expf(-x)); }
// logistic for values that leave as 16-bit (T = bf16): hardware exp and reciprocal; accurate for T = float
template <typename T>
__device__ __forceinline__ float logistic_for(float x) {
    if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(1.f + __expf(-x));
    else return logistic(x);
}
__device__ __forceinline__ float softplus(float x) { return x > 30.f ? x : log1pf(expf(x)); }

// tanh form of gelu: z times the logistic of 2 sqrt(2 / pi) (z + 0.044715 z^3)
template <typename T>
__device__ __forceinline__ float gelu_tanh(float z) {
    return z * logistic_for<T>(1.5957691216057308f * (z + 0.044715f * z * z * z));
}


static inline int ceil_div(int a, int b) { return (a + b - 1) / b; }

// Columns [at, at + n) of a projection's slabs through gelu into rows out + t * ldo (n = 0: nothing): a job that kernels
// with few rows take along in blocks of their own.
struct GeluJob {
    int at, n, ldo;
    void* out;
};

template <bool PARTS, typename T>
__device__ __forceinline__ void gelu_piece(const ProjSrc& src, const GeluJob& j, int t, int c) {
    if (c >= j.n) return;
    float v[8];
    proj8<PARTS>(src, t, j.at + c, v);
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = gelu_tanh<T>(v[k]);
    store8(reinterpret_cast<T*>(j.out) + (size_t)t * j.ldo + c, v);
}

static inline bool gelu_job_ok(const GeluJob& j, int S, int ld) {
    return j.n == 0 || (S >= 1 && j.n > 0 && j.out && j.at >= 0 && j.at % 8 == 0 && j.n % 8 == 0 && j.ldo % 8 == 0 && j.at + j.n <= ld);
}
