// Chunked gated delta rule on MFMA (prompt portions, 16-bit activations): the recurrence of delta.hip's delta_step over
// chunks of 64 tokens in matrix form.  With c_i the running sum of the log2 decays over the chunk, k_i and q_i the
// convolved rows and rk_i, rq_i the factors that make them unit vectors (q's with dim^-1/2), per head
//
//   A[i][j] = beta_i 2^(c_i - c_j) rk_i rk_j (k_i . k_j)  (j < i)     T = (I + A)^-1 diag(beta)
//   M[i][j] = 2^(c_i - c_j) rq_i rk_j (q_i . k_j)         (j <= i)
//   U = T (V - diag(2^c rk) K S)       O = diag(2^c rq) Q S + M U      S <- 2^(c_last) S + K^T diag(2^(c_last - c) rk) U
//
// delta_prep computes T and M of every chunk (parallel over chunks): dot products of 16-bit rows on MFMA, the unit lower
// triangular inverse in fp32 -- 16 x 16 diagonal blocks by substitution, then blocks merged with fp32 MFMA products.
// delta_chunk walks the chunks.  Value columns are independent throughout, so a wave owns 16 of them: its state block is
// in accumulator registers, and every product's fp32 result tile is the next product's operand as it stands (the other
// operand's columns are read in the order the tile has), so nothing but k, q and v passes through LDS.
//
// k, q and v are 16-bit operands (exact); everything fp32 -- T, M, S, the right-hand sides, U -- enters a product as two
// bf16 terms (hi + lo), accumulated in fp32.
#include "delta.h"

namespace {
constexpr int Q = 64;
constexpr float LOG2E = 1.4426950408889634f;
constexpr int FR = 6;                  // lower-triangular 16 x 32 operand tiles of a 64 x 64 matrix
constexpr int FRAGS = 4 * FR * 64;     // operand pieces (16 bytes) of one (chunk, head): T hi, T lo, M hi, M lo
typedef short s4 __attribute__((ext_vector_type(4)));
typedef short s8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) s4 lds_s4;

__device__ __forceinline__ s4 tr4(const bf16* p) { return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)p); }
__device__ __forceinline__ bf16x8 join(s4 a, s4 b) {
    return __builtin_bit_cast(bf16x8, (s8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]}));
}
__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma32(float a, float b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ void split(f32x4 a, f32x4 b, bf16x8& hi, bf16x8& lo) {
    u32x4 h, l;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const float x = j < 2 ? a[2 * j] : b[2 * j - 4], y = j < 2 ? a[2 * j + 1] : b[2 * j - 3];
        h[j] = pack2(x, y);
        l[j] = pack2(x - __uint_as_float(h[j] << 16), y - __uint_as_float(h[j] & 0xffff0000u));
    }
    hi = __builtin_bit_cast(bf16x8, h);
    lo = __builtin_bit_cast(bf16x8, l);
}
__device__ __forceinline__ int frag_of(int ib, int jp) { return ib < 2 ? ib : 2 * (ib - 1) + jp; }

// c += L b for a lower-triangular 64 x 64 L given as operand tiles (hi, then lo), b as operands (hi, lo) or as four
// accumulator tiles
__device__ __forceinline__ void lower(f32x4* c, const uint4* l, const bf16x8* hi, const bf16x8* lo) {
#pragma unroll
    for (int jp = 0; jp < 2; ++jp) {
#pragma unroll
        for (int ib = 2 * jp; ib < 4; ++ib) c[ib] = mma(__builtin_bit_cast(bf16x8, l[frag_of(ib, jp)]), hi[jp], c[ib]);
#pragma unroll
        for (int ib = 2 * jp; ib < 4; ++ib) c[ib] = mma(__builtin_bit_cast(bf16x8, l[frag_of(ib, jp)]), lo[jp], c[ib]);
#pragma unroll
        for (int ib = 2 * jp; ib < 4; ++ib) c[ib] = mma(__builtin_bit_cast(bf16x8, l[FR + frag_of(ib, jp)]), hi[jp], c[ib]);
    }
}
__device__ __forceinline__ void lower(f32x4* c, const uint4* l, const f32x4* b) {
    bf16x8 hi[2], lo[2];
    split(b[0], b[1], hi[0], lo[0]);
    split(b[2], b[3], hi[1], lo[1]);
    lower(c, l, hi, lo);
}
}  // namespace

// x: convolved rows.  chunks: (first row, end row) of every chunk.  Per (chunk, head): frags [FRAGS] 16-byte pieces,
// vec [3][64] = 2^c rk | 2^c rq | 2^(c_last - c) rk and 2^(c_last) at [3][0] (stride 256 floats).
template <int NB>
__global__ __launch_bounds__(256, NB <= 4 ? 4 : 2) void delta_prep_kernel(const bf16* __restrict__ x, DeltaArgs a,
                                                         const int2* __restrict__ chunks, uint4* __restrict__ frags,
                                                         float* __restrict__ vec) {
    constexpr int NN = 32 * NB, LK = NN + 16, LA = Q + 4;
    // the rows' place is taken over by A and T once their dot products are in registers
    constexpr int ROWS_B = 2 * 2 * Q * LK, AT_B = 2 * 4 * Q * LA;
    __shared__ __attribute__((aligned(16))) char pool[ROWS_B > AT_B ? ROWS_B : AT_B];
    bf16* sK = reinterpret_cast<bf16*>(pool);
    bf16* sQ = sK + Q * LK;
    float* sA = reinterpret_cast<float*>(pool);
    float* sT = sA + Q * LA;
    __shared__ __attribute__((aligned(16))) float s_c[Q], s_beta[Q], s_rk[Q], s_rq[Q];
    const int kh = blockIdx.x, ck = blockIdx.y;
    const int2 ch = chunks[ck];
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    // raw decays and step sizes of a head's 64 tokens (wave 0), fetched a head ahead
    float ar = 0.f, br = 0.f;
    const int rep = a.heads / a.kv_heads, tok = min(ch.x + lane, ch.y - 1);
#define LOAD_RAW(HEAD)                                                                                          \
    if (w == 0) {                                                                                               \
        ar = a.u.S ? proj_at<true>(a.u, tok, a.a_at + (HEAD)) : proj_at<false>(a.u, tok, a.a_at + (HEAD));      \
        br = a.u.S ? proj_at<true>(a.u, tok, a.b_at + (HEAD)) : proj_at<false>(a.u, tok, a.b_at + (HEAD));      \
    }
    LOAD_RAW(kh * rep)
    for (int i = tid; i < Q * 4 * NB; i += 256) {
        const int row = i / (4 * NB), n = 8 * (i % (4 * NB)), t = ch.x + row;
        u32x4 k = {0, 0, 0, 0}, q = {0, 0, 0, 0};
        if (t < ch.y && n < a.N) {
            const bf16* p = x + (size_t)t * a.ldx + kh * a.N + n;
            q = *reinterpret_cast<const u32x4*>(p);
            k = *reinterpret_cast<const u32x4*>(p + a.xk);
        }
        *reinterpret_cast<u32x4*>(sK + row * LK + n) = k;
        *reinterpret_cast<u32x4*>(sQ + row * LK + n) = q;
    }
    __syncthreads();
    {  // unit-vector factors: four lanes a row
        const int row = tid >> 2;
        float kk = 0.f, qq = 0.f;
        for (int c = 8 * (tid & 3); c < NN; c += 32) {
            float f[8];
            unpack8(*reinterpret_cast<const uint4*>(sK + row * LK + c), f);
#pragma unroll
            for (int j = 0; j < 8; ++j) kk += f[j] * f[j];
            unpack8(*reinterpret_cast<const uint4*>(sQ + row * LK + c), f);
#pragma unroll
            for (int j = 0; j < 8; ++j) qq += f[j] * f[j];
        }
        kk += __shfl_xor(kk, 1, 64); kk += __shfl_xor(kk, 2, 64);
        qq += __shfl_xor(qq, 1, 64); qq += __shfl_xor(qq, 2, 64);
        if ((tid & 3) == 0) {
            s_rk[row] = 1.f / sqrtf(kk + 1e-6f);
            s_rq[row] = a.q_scale / sqrtf(qq + 1e-6f);
        }
    }
    // (k_j . k_i) and (k_j . q_i): lane holds i = 16 w + r16, j = 16 jb + 4 g + e
    f32x4 gk[4], gq[4];
    {
        bf16x8 ki[NB], qi[NB];
#pragma unroll
        for (int kb = 0; kb < NB; ++kb) {
            ki[kb] = *reinterpret_cast<const bf16x8*>(sK + (16 * w + r16) * LK + 32 * kb + 8 * g);
            qi[kb] = *reinterpret_cast<const bf16x8*>(sQ + (16 * w + r16) * LK + 32 * kb + 8 * g);
        }
#pragma unroll
        for (int jb = 0; jb < 4; ++jb) {
            gk[jb] = gq[jb] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (jb <= w) {
#pragma unroll
                for (int kb = 0; kb < NB; ++kb) {
                    const bf16x8 kj = *reinterpret_cast<const bf16x8*>(sK + (16 * jb + r16) * LK + 32 * kb + 8 * g);
                    gk[jb] = mma(kj, ki[kb], gk[jb]);
                    gq[jb] = mma(kj, qi[kb], gq[jb]);
                }
            }
        }
    }
    const int i = 16 * w + r16;
    for (int hr = 0; hr < rep; ++hr) {
        const int head = kh * rep + hr;
        __syncthreads();  // factors ready; the previous head's readers are done
        if (w == 0) {
            const int t = ch.x + lane;
            float c = 0.f, beta = 0.f;
            if (t < ch.y) {
                beta = logistic(br);
                c = a.a_neg[head] * LOG2E * softplus(ar + a.dt_bias[head]);
            }
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const float v = __shfl_up(c, o, 64);
                if (lane >= o) c += v;
            }
            s_c[lane] = c;
            s_beta[lane] = beta;
            const float last = __shfl(c, 63, 64), e = __builtin_amdgcn_exp2f(c), rk = s_rk[lane];
            float* v = vec + ((size_t)ck * a.heads + head) * 256;
            v[lane] = e * rk;
            v[64 + lane] = e * s_rq[lane];
            v[128 + lane] = __builtin_amdgcn_exp2f(last - c) * rk;
            if (lane == 0) v[192] = __builtin_amdgcn_exp2f(last);
        }
        if (hr + 1 < rep) LOAD_RAW(head + 1)
        __syncthreads();
        uint4* fr = frags + ((size_t)ck * a.heads + head) * FRAGS;
        const float ci = s_c[i], bi = s_beta[i] * s_rk[i], qi = s_rq[i];
        f32x4 m[4];
#pragma unroll
        for (int jb = 0; jb < 4; ++jb) {
            m[jb] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (jb <= w) {
                const int j0 = 16 * jb + 4 * g;
                const f32x4 cj = *reinterpret_cast<const f32x4*>(s_c + j0), rj = *reinterpret_cast<const f32x4*>(s_rk + j0);
                f32x4 av;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float d = j0 + e <= i ? __builtin_amdgcn_exp2f(ci - cj[e]) * rj[e] : 0.f;
                    m[jb][e] = d * qi * gq[jb][e];
                    av[e] = j0 + e < i ? d * bi * gk[jb][e] : 0.f;
                }
                *reinterpret_cast<f32x4*>(sA + i * LA + j0) = av;
            }
        }
#pragma unroll
        for (int jp = 0; jp < 2; ++jp)
            if (jp <= (w >> 1)) {
                bf16x8 hi, lo;
                split(m[2 * jp], m[2 * jp + 1], hi, lo);
                const int f = frag_of(w, jp) * 64 + lane;
                fr[2 * FR * 64 + f] = __builtin_bit_cast(uint4, hi);
                fr[3 * FR * 64 + f] = __builtin_bit_cast(uint4, lo);
            }
        __syncthreads();
        {  // diagonal block w: column r16 of its inverse by substitution (lane groups do the same work)
            int ab = 16 * w * LA + 16 * w;
            float xv[16];
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                float s = r == r16 ? 1.f : 0.f;
#pragma unroll
                for (int l = 0; l < r; ++l) s -= sA[ab + r * LA + l] * xv[l];
                xv[r] = s;
                // rows are read two at a time: all of them read ahead would fill the register file
                if (r & 1) asm volatile("" : "+v"(ab), "+v"(xv[r]));
            }
#pragma unroll
            for (int r = 0; r < 16; ++r)
                if ((r >> 2) == g) sT[(16 * w + r) * LA + 16 * w + r16] = xv[r];
        }
        __syncthreads();
        if (w < 2) {  // blocks (1, 0) and (3, 2): -T A T
            const int o = 32 * w;
            const f32x4 aa = *reinterpret_cast<const f32x4*>(sA + (o + 16 + r16) * LA + o + 4 * g);
            const f32x4 tt = *reinterpret_cast<const f32x4*>(sT + (o + 16 + r16) * LA + o + 16 + 4 * g);
            f32x4 X = {0.f, 0.f, 0.f, 0.f}, Y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int e = 0; e < 4; ++e) X = mma32(aa[e], sT[(o + 4 * g + e) * LA + o + r16], X);
#pragma unroll
            for (int e = 0; e < 4; ++e) Y = mma32(tt[e], X[e], Y);
#pragma unroll
            for (int e = 0; e < 4; ++e) sT[(o + 16 + 4 * g + e) * LA + o + r16] = -Y[e];
        }
        __syncthreads();
        if (w < 2) {  // the lower left 32 x 32 block, columns [16 w, 16 w + 16)
            f32x4 X[2], Y[2];
#pragma unroll
            for (int ib = 0; ib < 2; ++ib) {
                X[ib] = Y[ib] = f32x4{0.f, 0.f, 0.f, 0.f};
                for (int l = w; l < 2; ++l) {
                    const f32x4 aa = *reinterpret_cast<const f32x4*>(sA + (32 + 16 * ib + r16) * LA + 16 * l + 4 * g);
#pragma unroll
                    for (int e = 0; e < 4; ++e) X[ib] = mma32(aa[e], sT[(16 * l + 4 * g + e) * LA + 16 * w + r16], X[ib]);
                }
            }
#pragma unroll
            for (int ib = 0; ib < 2; ++ib)
#pragma unroll
                for (int l = 0; l <= ib; ++l) {
                    const f32x4 tt = *reinterpret_cast<const f32x4*>(sT + (32 + 16 * ib + r16) * LA + 32 + 16 * l + 4 * g);
#pragma unroll
                    for (int e = 0; e < 4; ++e) Y[ib] = mma32(tt[e], X[l][e], Y[ib]);
                }
#pragma unroll
            for (int ib = 0; ib < 2; ++ib)
#pragma unroll
                for (int e = 0; e < 4; ++e) sT[(32 + 16 * ib + 4 * g + e) * LA + 16 * w + r16] = -Y[ib][e];
        }
        __syncthreads();
#pragma unroll
        for (int jp = 0; jp < 2; ++jp)
            if (jp <= (w >> 1)) {
                f32x4 t[2];
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const int j0 = 32 * jp + 16 * h + 4 * g;
                    t[h] = f32x4{0.f, 0.f, 0.f, 0.f};
                    if (2 * jp + h <= w)
                        t[h] = *reinterpret_cast<const f32x4*>(sT + i * LA + j0) * *reinterpret_cast<const f32x4*>(s_beta + j0);
                }
                bf16x8 hi, lo;
                split(t[0], t[1], hi, lo);
                const int f = frag_of(w, jp) * 64 + lane;
                fr[f] = __builtin_bit_cast(uint4, hi);
                fr[FR * 64 + f] = __builtin_bit_cast(uint4, lo);
            }
    }
}

#undef LOAD_RAW

// Rows of k and q in LDS.  128 and 256 wide: unpadded, 16-byte pieces exchanged by a row-dependent mask, so that the 16 rows
// of a read lie in different banks; narrower: padded to the same end.
template <int NB>
constexpr int row_stride() { return NB >= 4 ? 32 * NB : 32 * NB + 8; }
template <int NB>
__device__ __forceinline__ int row_at(int row, int col) {
    if constexpr (NB >= 4) return row * 32 * NB + (col ^ ((((row & 3) << 2) | ((row >> 2) & 3)) << 3));
    return row * row_stride<NB>() + col;
}
// Rows 4 g + e of state tile nb are this dimension plus e: the tiles of a pair take turns in fours, so that a lane's operand
// of the products over the state is eight neighbouring columns of a row.
__device__ __forceinline__ int tile_row(int nb, int g) { return 32 * (nb >> 1) + 8 * g + 4 * (nb & 1); }

// Staging of a chunk through the registers of NTH threads.  Loads are unconditional, so that later waits can count them: rows
// past the segment and columns past the head repeat valid ones, and are zeroed on the way into LDS.  Addresses are a uniform
// base and a 32-bit offset.
#define LOAD_CHUNK(T0, CK)                                                                                  \
    {                                                                                                       \
        const size_t row0_ = (size_t)(T0) * a.ldx;                                                          \
        const int last_ = re - 1 - (T0);                                                                    \
        _Pragma("unroll") for (int i = 0; i < KIT; ++i) {                                                   \
            const int idx = tid + NTH * i, n = min(8 * (idx % (4 * NB)), a.N - 8);                          \
            const uint32_t at_ = 2u * (uint32_t)(min(idx / (4 * NB), last_) * a.ldx + n);                   \
            kreg[i] = *reinterpret_cast<const u32x4*>(reinterpret_cast<const char*>(kcol + row0_) + at_);   \
            qreg[i] = *reinterpret_cast<const u32x4*>(reinterpret_cast<const char*>(qcol + row0_) + at_);   \
        }                                                                                                   \
        _Pragma("unroll") for (int i = 0; i < VR; ++i) {                                                     \
            const int idx = tid + NTH * i, c = min(8 * (idx % (2 * WPB)), a.P - 8 - pb);                    \
            const uint32_t at_ = 2u * (uint32_t)(min(idx / (2 * WPB), last_) * a.ldx + c);                  \
            vreg[i] = *reinterpret_cast<const u32x4*>(reinterpret_cast<const char*>(vcol + row0_) + at_);   \
        }                                                                                                   \
        const float* vs_ = vec + ((size_t)(CK) * a.heads + head) * 256;                                     \
        _Pragma("unroll") for (int i = 0; i < VIT; ++i) vecr[i] = vs_[min(tid + NTH * i, 192)];             \
    }
#define STORE_CHUNK(T0)                                                                                     \
    {                                                                                                       \
        if ((T0) + Q > re || a.N < NN || pb + 16 * WPB > a.P) {                                             \
            const u32x4 zero = {0, 0, 0, 0};                                                                \
            _Pragma("unroll") for (int i = 0; i < KIT; ++i) {                                               \
                const int idx = tid + NTH * i;                                                              \
                const bool on = (T0) + idx / (4 * NB) < re && 8 * (idx % (4 * NB)) < a.N;                   \
                kreg[i] = on ? kreg[i] : zero;                                                              \
                qreg[i] = on ? qreg[i] : zero;                                                              \
            }                                                                                               \
            _Pragma("unroll") for (int i = 0; i < VR; ++i) {                                                 \
                const int idx = tid + NTH * i;                                                              \
                const bool on = (T0) + idx / (2 * WPB) < re && pb + 8 * (idx % (2 * WPB)) < a.P;            \
                vreg[i] = on ? vreg[i] : zero;                                                              \
            }                                                                                               \
        }                                                                                                   \
        _Pragma("unroll") for (int i = 0; i < KIT; ++i) {                                                   \
            const int idx = tid + NTH * i, o_ = row_at<NB>(idx / (4 * NB), 8 * (idx % (4 * NB)));           \
            if (KIT * NTH == Q * 4 * NB || idx < Q * 4 * NB) {                                              \
                *reinterpret_cast<u32x4*>(sK + o_) = kreg[i];                                               \
                *reinterpret_cast<u32x4*>(sQ + o_) = qreg[i];                                               \
            }                                                                                               \
        }                                                                                                   \
        _Pragma("unroll") for (int i = 0; i < VR; ++i) {                                                     \
            const int idx = tid + NTH * i;                                                                  \
            *reinterpret_cast<u32x4*>(sV + idx / (2 * WPB) * LV + 8 * (idx % (2 * WPB))) = vreg[i];         \
        }                                                                                                   \
        _Pragma("unroll") for (int i = 0; i < VIT; ++i)                                                     \
            if (NTH <= 256 || tid + NTH * i < 256) s_vec[tid + NTH * i] = vecr[i];                          \
    }

// o: output tiles of the chunk at t0
#define STORE_ROWS(o)                    \
    if (p < a.P) {                                                                                          \
        float* yb = y + (size_t)(t0 - y0) * inner + head * a.P;                                             \
        const uint32_t yo = 4u * (uint32_t)(4 * g * inner + p);                                             \
        const int left = re - t0 - 4 * g;                                                                   \
        if (t0 + Q <= re) {                                                                                 \
            _Pragma("unroll") for (int ib = 0; ib < 4; ++ib)                                                \
                _Pragma("unroll") for (int e = 0; e < 4; ++e)                                               \
                    *reinterpret_cast<float*>(reinterpret_cast<char*>(yb + (size_t)(16 * ib + e) * inner) + yo) = o[ib][e];\
        } else {                                                                                            \
            _Pragma("unroll") for (int ib = 0; ib < 4; ++ib)                                                \
                _Pragma("unroll") for (int e = 0; e < 4; ++e)                                               \
                    if (16 * ib + e < left)                                                                 \
                        *reinterpret_cast<float*>(reinterpret_cast<char*>(yb + (size_t)(16 * ib + e) * inner) + yo) = o[ib][e];\
        }                                                                                                   \
    }

// Grid (heads, blocks of 16 WPB value columns, segments): heads first, so that the blocks of a head, which read the same
// operands, share an XCD's L2.  segs: (segment, first row, end row, first chunk).
template <int NB, int WPB>
__global__ __launch_bounds__(64 * WPB, 1) void delta_chunk_kernel(const bf16* __restrict__ x, DeltaArgs a,
                                                                  const int4* __restrict__ segs,
                                                                  const int* __restrict__ slots,
                                                                  const int* __restrict__ pos0,
                                                                  const uint4* __restrict__ frags,
                                                                  const float* __restrict__ vec,
                                                                  float* __restrict__ state, float* __restrict__ y,
                                                                  int y0) {
    constexpr int NTH = 64 * WPB, NN = 32 * NB, LK = row_stride<NB>(), LV = 16 * WPB + 16, NT = 2 * NB, GN = NT < 4 ? NT : 4;
    constexpr int KIT = (Q * 4 * NB + NTH - 1) / NTH, VR = 2;  // staging rounds of k and of q, of v
    constexpr int VIT = NTH < 256 ? 256 / NTH : 1;
    __shared__ __attribute__((aligned(16))) bf16 sK[Q * LK];
    __shared__ __attribute__((aligned(16))) bf16 sQ[Q * LK];
    __shared__ __attribute__((aligned(16))) bf16 sV[Q * LV];
    __shared__ __attribute__((aligned(16))) float s_vec[256];
    const int head = blockIdx.x, pb = 16 * WPB * blockIdx.y;
    const int4 sg = segs[blockIdx.z];
    const int rb = sg.y, re = sg.z;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4, q4 = r16 >> 2, p4 = 4 * (r16 & 3);
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int kh = head / (a.heads / a.kv_heads), inner = a.heads * a.P;
    const bf16* qcol = x + kh * a.N;
    const bf16* kcol = qcol + a.xk;
    const bf16* vcol = x + a.xv + head * a.P + pb;
    const int p = pb + 16 * w + r16;  // this lane's value column
    u32x4 kreg[KIT], qreg[KIT], vreg[VR];
    float vecr[VIT];
    // state tiles: rows tile_row(nb, g) + e, column p
    float* st_p = state + ((size_t)slots[sg.x] * a.heads + head) * a.P * a.N4 + (size_t)p * a.N4;
    f32x4 st[NT];
    const bool cont = pos0[sg.x] > 0;
#pragma unroll
    for (int nb = 0; nb < NT; ++nb) {
        st[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int n = tile_row(nb, g);
        if (cont && p < a.P && n < a.N) st[nb] = *reinterpret_cast<const f32x4*>(st_p + n);
    }
    LOAD_CHUNK(rb, sg.w)
    STORE_CHUNK(rb)
    __syncthreads();
    int ck = sg.w;
    for (int t0 = rb; t0 < re; t0 += Q, ++ck) {
        const bool more = t0 + Q < re;
        const uint4* fr = frags + ((size_t)ck * a.heads + head) * FRAGS + lane;
        uint4 tf[2 * FR];
#pragma unroll
        for (int f = 0; f < 2 * FR; ++f) tf[f] = fr[64 * f];
        __builtin_amdgcn_sched_barrier(0);  // loads stay here
        // products run over independent accumulators: no MFMA waits for the one before it
        f32x4 r[4], o[4];
#pragma unroll
        for (int ib = 0; ib < 4; ++ib) r[ib] = o[ib] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < NB; ++kb) {
            bf16x8 sh, sl, kf[4], qf[4];
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) {
                const int at = row_at<NB>(r16, 32 * kb + 8 * g) + 16 * ib * LK;
                kf[ib] = *reinterpret_cast<const bf16x8*>(sK + at);
                qf[ib] = *reinterpret_cast<const bf16x8*>(sQ + at);
            }
            split(st[2 * kb], st[2 * kb + 1], sh, sl);
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) {
                r[ib] = mma(kf[ib], sh, r[ib]);
                o[ib] = mma(qf[ib], sh, o[ib]);
            }
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) {
                r[ib] = mma(kf[ib], sl, r[ib]);
                o[ib] = mma(qf[ib], sl, o[ib]);
            }
        }
#pragma unroll
        for (int ib = 0; ib < 4; ++ib) {
            const f32x4 ek = *reinterpret_cast<const f32x4*>(s_vec + 16 * ib + 4 * g);
            const f32x4 eq = *reinterpret_cast<const f32x4*>(s_vec + 64 + 16 * ib + 4 * g);
            const s4 vt = tr4(sV + (16 * ib + 4 * g + q4) * LV + 16 * w + p4);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                r[ib][e] = __uint_as_float((uint32_t)(uint16_t)vt[e] << 16) - ek[e] * r[ib][e];
                o[ib][e] *= eq[e];
            }
        }
        f32x4 u[4];
#pragma unroll
        for (int ib = 0; ib < 4; ++ib) u[ib] = f32x4{0.f, 0.f, 0.f, 0.f};
        lower(u, tf, r);
#pragma unroll
        for (int f = 0; f < 2 * FR; ++f) tf[f] = fr[64 * (2 * FR + f)];  // M
        LOAD_CHUNK(more ? t0 + Q : t0, more ? ck + 1 : ck)
        __builtin_amdgcn_sched_barrier(0);  // loads stay here
        {  // state
            const float dec = s_vec[192];
            bf16x8 wh[2], wl[2];
#pragma unroll
            for (int jp = 0; jp < 2; ++jp) {
                const f32x4 w0 = *reinterpret_cast<const f32x4*>(s_vec + 128 + 32 * jp + 4 * g);
                const f32x4 w1 = *reinterpret_cast<const f32x4*>(s_vec + 128 + 32 * jp + 16 + 4 * g);
                split(u[2 * jp] * w0, u[2 * jp + 1] * w1, wh[jp], wl[jp]);
            }
#pragma unroll
            for (int nb = 0; nb < NT; ++nb) st[nb] *= dec;
#pragma unroll
            for (int n4 = 0; n4 < NT; n4 += GN) {
#pragma unroll
                for (int jp = 0; jp < 2; ++jp) {
                    bf16x8 kt[GN];
#pragma unroll
                    for (int i = 0; i < GN; ++i) {
                        const bf16* kr = sK + row_at<NB>(4 * g + q4, tile_row(n4 + i, r16 & 3)) + 32 * jp * LK;
                        kt[i] = join(tr4(kr), tr4(kr + 16 * LK));
                    }
#pragma unroll
                    for (int i = 0; i < GN; ++i) st[n4 + i] = mma(kt[i], wh[jp], st[n4 + i]);
#pragma unroll
                    for (int i = 0; i < GN; ++i) st[n4 + i] = mma(kt[i], wl[jp], st[n4 + i]);
                }
            }
        }
        lower(o, tf, u);
        STORE_ROWS(o)
        if (more) {
            __syncthreads();  // every wave is done with this chunk's LDS images
            STORE_CHUNK(t0 + Q)
            __syncthreads();
        }
    }
    if (p < a.P) {
#pragma unroll
        for (int nb = 0; nb < NT; ++nb)
            if (tile_row(nb, g) < a.N) *reinterpret_cast<f32x4*>(st_p + tile_row(nb, g)) = st[nb];
    }
}

// The same with two waves per 16 value columns, for grids that leave SIMDs idle: one carries the state (its chain is what a
// chunk takes), the other turns the state at the chunk's start and U into output rows beside it.  Both reach it as finished
// operands through LDS.
template <int NB, int WPB>
__global__ __launch_bounds__(128 * WPB, 1) void delta_chunk_pair_kernel(const bf16* __restrict__ x, DeltaArgs a,
                                                                        const int4* __restrict__ segs,
                                                                        const int* __restrict__ slots,
                                                                        const int* __restrict__ pos0,
                                                                        const uint4* __restrict__ frags,
                                                                        const float* __restrict__ vec,
                                                                        float* __restrict__ state, float* __restrict__ y,
                                                                        int y0) {
    constexpr int NTH = 128 * WPB, NN = 32 * NB, LK = row_stride<NB>(), LV = 16 * WPB + 16, NT = 2 * NB, GN = NT < 4 ? NT : 4;
    constexpr int KIT = (Q * 4 * NB + NTH - 1) / NTH, VR = 1;
    constexpr int VIT = NTH < 256 ? 256 / NTH : 1;
    __shared__ __attribute__((aligned(16))) bf16 sK[Q * LK];
    __shared__ __attribute__((aligned(16))) bf16 sQ[Q * LK];
    __shared__ __attribute__((aligned(16))) bf16 sV[Q * LV];
    __shared__ __attribute__((aligned(16))) float s_vec[256];
    __shared__ bf16x8 sS[WPB][2 * NB][64];  // state operands, hi and lo
    __shared__ bf16x8 sU[WPB][4][64];       // U operands, hi and lo
    const int head = blockIdx.x, pb = 16 * WPB * blockIdx.y;
    const int4 sg = segs[blockIdx.z];
    const int rb = sg.y, re = sg.z;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4, q4 = r16 >> 2, p4 = 4 * (r16 & 3);
    const int wv = __builtin_amdgcn_readfirstlane(tid >> 6), w = wv % WPB;
    const int kh = head / (a.heads / a.kv_heads), inner = a.heads * a.P;
    const bf16* qcol = x + kh * a.N;
    const bf16* kcol = qcol + a.xk;
    const bf16* vcol = x + a.xv + head * a.P + pb;
    const int p = pb + 16 * w + r16;  // this lane's value column
    u32x4 kreg[KIT], qreg[KIT], vreg[VR];
    float vecr[VIT];
    const uint4* fr = frags + ((size_t)sg.w * a.heads + head) * FRAGS + lane;  // this chunk's T and M
    const size_t fr_step = (size_t)a.heads * FRAGS;
    uint4 lf[2 * FR];
    int ck = sg.w;
    if (wv < WPB) {
        float* st_p = state + ((size_t)slots[sg.x] * a.heads + head) * a.P * a.N4 + (size_t)p * a.N4;
        f32x4 st[NT];
        const bool cont = pos0[sg.x] > 0;
#pragma unroll
        for (int nb = 0; nb < NT; ++nb) {
            st[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
            const int n = tile_row(nb, g);
            if (cont && p < a.P && n < a.N) st[nb] = *reinterpret_cast<const f32x4*>(st_p + n);
        }
        bf16x8 sh[NB], sl[NB];
#define PUBLISH()                                                         \
    _Pragma("unroll") for (int kb = 0; kb < NB; ++kb) {                   \
        split(st[2 * kb], st[2 * kb + 1], sh[kb], sl[kb]);                \
        sS[w][kb][lane] = sh[kb];                                         \
        sS[w][NB + kb][lane] = sl[kb];                                    \
    }
#pragma unroll
        for (int f = 0; f < 2 * FR; ++f) lf[f] = fr[64 * f];
        LOAD_CHUNK(rb, ck)
        STORE_CHUNK(rb)
        PUBLISH()
        __syncthreads();
        for (int t0 = rb; t0 < re; t0 += Q) {
            const bool more = t0 + Q < re;
            LOAD_CHUNK(more ? t0 + Q : t0, more ? ck + 1 : ck)
            __builtin_amdgcn_sched_barrier(0);  // loads stay here
            f32x4 r[4], u[4];
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) r[ib] = u[ib] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kb = 0; kb < NB; ++kb) {
                bf16x8 kf[4];
#pragma unroll
                for (int ib = 0; ib < 4; ++ib)
                    kf[ib] = *reinterpret_cast<const bf16x8*>(sK + row_at<NB>(r16, 32 * kb + 8 * g) + 16 * ib * LK);
#pragma unroll
                for (int ib = 0; ib < 4; ++ib) r[ib] = mma(kf[ib], sh[kb], r[ib]);
#pragma unroll
                for (int ib = 0; ib < 4; ++ib) r[ib] = mma(kf[ib], sl[kb], r[ib]);
            }
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) {
                const f32x4 ek = *reinterpret_cast<const f32x4*>(s_vec + 16 * ib + 4 * g);
                const s4 vt = tr4(sV + (16 * ib + 4 * g + q4) * LV + 16 * w + p4);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    r[ib][e] = __uint_as_float((uint32_t)(uint16_t)vt[e] << 16) - ek[e] * r[ib][e];
            }
            lower(u, lf, r);
            {
                bf16x8 h, l;
#pragma unroll
                for (int jp = 0; jp < 2; ++jp) {
                    split(u[2 * jp], u[2 * jp + 1], h, l);
                    sU[w][jp][lane] = h;
                    sU[w][2 + jp][lane] = l;
                }
            }
            __syncthreads();  // U is in LDS; the output waves have read the state
            if (more) fr += fr_step;
#pragma unroll
            for (int f = 0; f < 2 * FR; ++f) lf[f] = fr[64 * f];
            const float dec = s_vec[192];
            bf16x8 wh[2], wl[2];
#pragma unroll
            for (int jp = 0; jp < 2; ++jp) {
                const f32x4 w0 = *reinterpret_cast<const f32x4*>(s_vec + 128 + 32 * jp + 4 * g);
                const f32x4 w1 = *reinterpret_cast<const f32x4*>(s_vec + 128 + 32 * jp + 16 + 4 * g);
                split(u[2 * jp] * w0, u[2 * jp + 1] * w1, wh[jp], wl[jp]);
            }
#pragma unroll
            for (int nb = 0; nb < NT; ++nb) st[nb] *= dec;
#pragma unroll
            for (int n4 = 0; n4 < NT; n4 += GN)
#pragma unroll
                for (int jp = 0; jp < 2; ++jp) {
                    bf16x8 kt[GN];
#pragma unroll
                    for (int i = 0; i < GN; ++i) {
                        const bf16* kr = sK + row_at<NB>(4 * g + q4, tile_row(n4 + i, r16 & 3)) + 32 * jp * LK;
                        kt[i] = join(tr4(kr), tr4(kr + 16 * LK));
                    }
#pragma unroll
                    for (int i = 0; i < GN; ++i) st[n4 + i] = mma(kt[i], wh[jp], st[n4 + i]);
#pragma unroll
                    for (int i = 0; i < GN; ++i) st[n4 + i] = mma(kt[i], wl[jp], st[n4 + i]);
                }
            if (more) {
                __syncthreads();  // every wave is done with this chunk's LDS images
                STORE_CHUNK(t0 + Q)
                PUBLISH()
                __syncthreads();
                ++ck;
            }
        }
#undef PUBLISH
        if (p < a.P) {
#pragma unroll
            for (int nb = 0; nb < NT; ++nb)
                if (tile_row(nb, g) < a.N) *reinterpret_cast<f32x4*>(st_p + tile_row(nb, g)) = st[nb];
        }
        return;
    }
    fr += 64 * 2 * FR;
#pragma unroll
    for (int f = 0; f < 2 * FR; ++f) lf[f] = fr[64 * f];
    LOAD_CHUNK(rb, ck)
    STORE_CHUNK(rb)
    __syncthreads();
    for (int t0 = rb; t0 < re; t0 += Q) {
        const bool more = t0 + Q < re;
        LOAD_CHUNK(more ? t0 + Q : t0, more ? ck + 1 : ck)
        __builtin_amdgcn_sched_barrier(0);  // loads stay here
        f32x4 o[4];
#pragma unroll
        for (int ib = 0; ib < 4; ++ib) o[ib] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < NB; ++kb) {
            const bf16x8 sh = sS[w][kb][lane], sl = sS[w][NB + kb][lane];
            bf16x8 qf[4];
#pragma unroll
            for (int ib = 0; ib < 4; ++ib)
                qf[ib] = *reinterpret_cast<const bf16x8*>(sQ + row_at<NB>(r16, 32 * kb + 8 * g) + 16 * ib * LK);
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) o[ib] = mma(qf[ib], sh, o[ib]);
#pragma unroll
            for (int ib = 0; ib < 4; ++ib) o[ib] = mma(qf[ib], sl, o[ib]);
        }
#pragma unroll
        for (int ib = 0; ib < 4; ++ib) o[ib] *= *reinterpret_cast<const f32x4*>(s_vec + 64 + 16 * ib + 4 * g);
        __syncthreads();  // U is in LDS; the state has been read
        {
            const bf16x8 hi[2] = {sU[w][0][lane], sU[w][1][lane]}, lo[2] = {sU[w][2][lane], sU[w][3][lane]};
            lower(o, lf, hi, lo);
        }
        if (more) fr += fr_step;
#pragma unroll
        for (int f = 0; f < 2 * FR; ++f) lf[f] = fr[64 * f];
        STORE_ROWS(o)
        if (more) {
            __syncthreads();  // every wave is done with this chunk's LDS images
            STORE_CHUNK(t0 + Q)
            __syncthreads();
            ++ck;
        }
    }
}
#undef LOAD_CHUNK
#undef STORE_CHUNK
#undef STORE_ROWS

// 16-byte pieces and floats of workspace per (chunk, head)
MRSUM_API int mrsum_delta_chunk_pieces() { return FRAGS; }

// Segments of ``segs`` (segment, first row, end row, first chunk); chunks (first row, end row) of at most 64 rows each, in
// order.  x [T][ldx] bf16; frags [n_chunks][heads][FRAGS] 16-byte pieces, vec [n_chunks][heads][256] fp32: workspace.
// y: fp32 rows [T - y0][heads * P] from row y0 on.  P % 8 == 0, N % 8 == 0, N <= 256.  wpb: waves of 16 value columns per
// block (2, 4, or up to N = 128 also 8); pair: two waves each (2 or 4, N <= 128).
MRSUM_API int mrsum_delta_chunk(const void* x, int ldx, int xk, int xv, const void* u, int S, int ld, int T, int b_at,
                                int a_at, const float* dt_bias, const float* a_neg, float* state, const int* slots,
                                const int* pos0, const void* segs, int n_segs, const void* chunks, int n_chunks, void* frags,
                                float* vec, float* y, int y0, int heads, int kv_heads, int P, int N, int wpb, int pair,
                                hipStream_t s) {
    if (T <= 0 || n_segs <= 0) return 0;
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || heads > 65535 || n_segs > 65535 || n_chunks > 65535 ||
        n_chunks < n_segs || P <= 0 || N <= 0 || P % 8 || N % 8 || N > 256 || ldx % 8 || xk % 8 || xv % 8 ||
        xk < kv_heads * N || xv < xk + kv_heads * N || ldx < xv + heads * P || b_at + heads > ld || a_at + heads > ld ||
        (wpb != 2 && wpb != 4 && (wpb != 8 || N > 128)) || (pair && (wpb == 8 || N > 128)))
        return (int)hipErrorInvalidValue;
    const DeltaArgs a{ProjSrc{u, S, (size_t)T * ld, ld}, b_at, a_at, 0, dt_bias, a_neg, nullptr, 0.f,
                      1.f / sqrtf((float)N), ldx, xk, xv, 0, 0, 0, heads, kv_heads, P, N, N};
    const dim3 g1(kv_heads, n_chunks), g2(heads, ceil_div(P, 16 * wpb), n_segs);
#define DC_P(NB_, W_)                                                                                                     \
    delta_chunk_pair_kernel<NB_, W_><<<g2, 128 * W_, 0, s>>>((const bf16*)x, a, (const int4*)segs, slots, pos0,              \
                                                            (const uint4*)frags, vec, state, y, y0)
#define DC_W(NB_, W_)                                                                                                     \
    delta_chunk_kernel<NB_, W_><<<g2, 64 * W_, 0, s>>>((const bf16*)x, a, (const int4*)segs, slots, pos0, (const uint4*)frags, \
                                                       vec, state, y, y0)
#define DC(NB_)                                                                                              \
    {                                                                                                        \
        delta_prep_kernel<NB_><<<g1, 256, 0, s>>>((const bf16*)x, a, (const int2*)chunks, (uint4*)frags, vec); \
        if constexpr (NB_ < 8) {                                                                             \
            if (wpb == 8) DC_W(NB_, 8);                                                                      \
            else if (wpb == 4 && pair) DC_P(NB_, 4);                                                              \
            else if (wpb == 2 && pair) DC_P(NB_, 2);                                                         \
        }                                                                                                    \
        if (wpb == 4 && !pair) DC_W(NB_, 4);                                                                 \
        else if (wpb == 2 && !pair) DC_W(NB_, 2);                                                            \
    }
    if (N <= 32) DC(1)
    else if (N <= 64) DC(2)
    else if (N <= 128) DC(4)
    else DC(8)
#undef DC
#undef DC_W
#undef DC_P
    return (int)hipGetLastError();
}
