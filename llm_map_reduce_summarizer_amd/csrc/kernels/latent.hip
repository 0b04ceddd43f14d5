// Latent attention around its attention kernels (latent_attn.hip, attn_rows.hip):
//
//   latent_prep     columns of the input projection -> normed query latents; normed latent | rotated key part of every
//                   token into the paged cache [pages][1][64][row], row = rank8 + rot8 (both padded to 8 columns)
//   head_product    y[t, h, :] = W_h x[t, h, :] per head: queries into the latent space (with their rotated part beside
//                   it, so a head's query has the form of a cached row) and weighted latent sums out of it; the input of
//                   the latter may be unmerged split-K partial sums, which are merged on the way in
//   latent_rope     rotated parts of query rows (prompt portions)
//   latent_gather   the cached rows of the sequences of a pass side by side
//
// Rotation tables are [positions][rot / 2] (cosine, sine) fp32.  Norms and rotations run in fp32.
#include "common.h"

namespace {
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

struct PrepArgs {
    int dq, nq, ldq;            // query latent: first column, width, row stride of the output
    int dkv, nkv, dkr, rot;     // own latents (dkv < 0: none): columns and widths
    int rank8, row;
    const float* qw;
    const float* kvw;
    float eps;
    const float2* cs;
    const int* positions;
    const int* seq_idx;
    const int* block_tables;
    int bt_stride, page;
};
}  // namespace

// One block per token, or (WAVE: many rows) one wave; a thread holds CH pieces of 8 columns (sections start at multiples of
// 8; their padding columns are zero in the projection).
template <bool PARTS, typename T, int CH, bool WAVE>
__global__ __launch_bounds__(WAVE ? 256 : 1024) void latent_prep_kernel(ProjSrc src, PrepArgs a, int rows, T* __restrict__ cq,
                                                                        T* __restrict__ cache, GeluJob job) {
    __shared__ float red[64];
    if constexpr (PARTS && !WAVE) {
        if (blockIdx.y) {
            gelu_piece<true, T>(src, job, blockIdx.x, 8 * ((blockIdx.y - 1) * blockDim.x + threadIdx.x));
            return;
        }
    }
    const int t = WAVE ? 4 * blockIdx.x + (threadIdx.x >> 6) : blockIdx.x;
    const int tid = WAVE ? threadIdx.x & 63 : threadIdx.x, nt = WAVE ? 64 : blockDim.x;
    if (WAVE && t >= rows) return;
    const int pq = (a.nq + 7) / 8, pk = a.dkv >= 0 ? (a.nkv + 7) / 8 : 0;
    float v[CH][8];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int p = tid + nt * i;
        if (p < pq + pk) {
            proj8<PARTS>(src, t, p < pq ? a.dq + 8 * p : a.dkv + 8 * (p - pq), v[i]);
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < 8; ++j) ss += v[i][j] * v[i][j];
            if (p < pq) sq += ss;
            else sk += ss;
        }
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if constexpr (!WAVE) {
        const int lane = tid & 63, nw = nt >> 6;
        if (lane == 0) { red[tid >> 6] = sq; red[32 + (tid >> 6)] = sk; }
        __syncthreads();
        sq = wave_sum(lane < nw ? red[lane] : 0.f);
        sk = wave_sum(lane < nw ? red[32 + lane] : 0.f);
    }
    const float qs = 1.f / sqrtf(sq / (float)a.nq + a.eps);
    T* qo = cq + (size_t)t * a.ldq;
    const int pos = a.positions[t];
    T* co = nullptr;
    float ks = 0.f;
    if (a.dkv >= 0) {
        ks = 1.f / sqrtf(sk / (float)a.nkv + a.eps);
        const int page = a.block_tables[(size_t)a.seq_idx[t] * a.bt_stride + pos / a.page];
        co = cache + ((size_t)page * a.page + pos % a.page) * a.row;
    }
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int p = tid + nt * i;
        if (p < pq + pk) {
            const bool isq = p < pq;
            const int c = 8 * (isq ? p : p - pq), n = isq ? a.nq : a.nkv;
            const float* w = isq ? a.qw : a.kvw;
            const float mul = isq ? qs : ks;
            if (c + 8 <= n) {
                float g[8];
                load8(w + c, g);
#pragma unroll
                for (int j = 0; j < 8; ++j) v[i][j] *= mul * g[j];
            } else {
#pragma unroll
                for (int j = 0; j < 8; ++j) v[i][j] *= c + j < n ? mul * w[c + j] : 0.f;
            }
            store8(isq ? qo + c : co + c, v[i]);
        }
    }
    for (int c = 8 * pq + tid; c < a.ldq; c += nt) qo[c] = (T)0.f;
    if (a.dkv < 0) return;
    const int half = a.rot / 2;
    for (int i = tid; i < half; i += nt) {
        const float x = proj_at<PARTS>(src, t, a.dkr + i), y = proj_at<PARTS>(src, t, a.dkr + half + i);
        const float2 cs = a.cs[(size_t)pos * half + i];
        co[a.rank8 + i] = (T)(x * cs.x - y * cs.y);
        co[a.rank8 + half + i] = (T)(y * cs.x + x * cs.y);
    }
    for (int c = a.rank8 + a.rot + tid; c < a.row; c += nt) co[c] = (T)0.f;
}

template <bool PARTS, typename T>
static int launch_prep(const ProjSrc& p, const PrepArgs& a, void* cq, void* cache, int rows, const GeluJob& job,
                       hipStream_t s) {
    const int pieces = (a.nq + 7) / 8 + (a.dkv >= 0 ? (a.nkv + 7) / 8 : 0);
    const int nt = std::min(1024, ceil_div(pieces, 64) * 64);
    const int ch = ceil_div(pieces, nt);
    const dim3 grid(rows, 1 + ceil_div(job.n / 8, nt));
#define LP(C) latent_prep_kernel<PARTS, T, C, false><<<grid, nt, 0, s>>>(p, a, rows, (T*)cq, (T*)cache, job)
#define LPW(C) latent_prep_kernel<PARTS, T, C, true><<<ceil_div(rows, 4), 256, 0, s>>>(p, a, rows, (T*)cq, (T*)cache, job)
    if (!PARTS && rows >= 1024 && pieces <= 256) {
        if (pieces <= 64) LPW(1);
        else if (pieces <= 128) LPW(2);
        else LPW(4);
    } else if (ch <= 1) LP(1);
    else if (ch <= 2) LP(2);
    else if (ch <= 4) LP(4);
    else return (int)hipErrorInvalidValue;
#undef LP
#undef LPW
    return (int)hipGetLastError();
}

// src: S = 0 bf16 rows [T][ld], S >= 1 fp32 slabs.  f32: cq / cache fp32 (slabs only), else bf16.  dkv < 0: query
// latents only.  g_n > 0: columns of the slabs through gelu besides (GeluJob).
MRSUM_API int mrsum_latent_prep(const void* src, int S, int ld, int T, int f32, void* cq, int ldq, void* cache, int dq,
                                int nq, int dkv, int nkv, int dkr, int rot, int rank8, int row, const float* qw,
                                const float* kvw, float eps, const void* cs, const int* positions, const int* seq_idx,
                                const int* block_tables, int bt_stride, int page, int g_at, int g_n, void* g_out,
                                int g_ldo, hipStream_t s) {
    if (T <= 0) return 0;
    const GeluJob job{g_at, g_n, g_ldo, g_out};
    if (!gelu_job_ok(job, S, ld)) return (int)hipErrorInvalidValue;
    if (nq <= 0 || dq % 8 || ld % 8 || ldq % 8 || ldq < (nq + 7) / 8 * 8 || (f32 && S < 1) || page <= 0 ||
        (dkv >= 0 && (nkv <= 0 || dkv % 8 || rot % 2 || rank8 < nkv || rank8 % 8 || row < rank8 + rot || row % 8)))
        return (int)hipErrorInvalidValue;
    const PrepArgs a{dq, nq, ldq, dkv, nkv, dkr, rot, rank8, row, qw, kvw, eps, (const float2*)cs, positions, seq_idx,
                     block_tables, bt_stride, page};
    const ProjSrc p{src, S, (size_t)T * ld, ld};
    if (f32) return launch_prep<true, float>(p, a, cq, cache, T, job, s);
    if (S) return launch_prep<true, bf16>(p, a, cq, cache, T, job, s);
    return launch_prep<false, bf16>(p, a, cq, cache, T, job, s);
}

// ------------------------------------------------------------------------------------------------ per-head products
namespace {
constexpr int HP_ROWS = 16, HP_COLS = 128;
constexpr int HM_ROWS = 4, HM_THREADS = 1024, HM_DEPTH = 4;  // merging form: depth up to 128 HM_DEPTH

struct HeadArgs {
    ProjSrc x;        // head h of row t: columns [h * xs, h * xs + xk); SPLITS: unused
    int xs, xk;
    const void* w;    // [H][N][K], zero past xk
    int N, K;
    void* out;        // head h of row t at columns [h * os, h * os + N) of rows of stride ldo
    int os, ldo;
    int rows, H;
    // rotated tail (rot > 0): columns [h * xs + rx, + rot) of x, turned, to columns [h * os + ro, + rot8) of out
    int rot, rot8, rx, ro;
    const float2* cs;
    const int* positions;
    // split-K partials [rows][H][S][xk] fp32 and (max, sum) [rows][H][S][2] in log2 units
    const float* po;
    const float* ml;
    int splits;
    int mrows;        // rows of a merging block, at most HM_ROWS
};
}  // namespace

// MODE 0: 16-bit rows, 1: fp32 slabs, 2: split-K partials (fewer rows and more threads a block: merging is a matter of
// loads in flight).  Grid (column blocks + (rot ? 1 : 0), H, row blocks).
template <typename T, int MODE>
__global__ __launch_bounds__(MODE == 2 ? HM_THREADS : 256) void head_product_kernel(const HeadArgs a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    T* sx = reinterpret_cast<T*>(smem);
    const int ROWS = MODE == 2 ? a.mrows : HP_ROWS;
    const int tid = threadIdx.x, h = blockIdx.y, r0 = blockIdx.z * ROWS;
    const int nr = min(ROWS, a.rows - r0);
    const int nb = (a.N + HP_COLS - 1) / HP_COLS;
    if ((int)blockIdx.x == nb) {
        if constexpr (MODE != 2) {
            const int half = a.rot / 2;
            T* out = reinterpret_cast<T*>(a.out);
            for (int i = tid; i < nr * half; i += 256) {
                const int t = r0 + i / half, c = i % half;
                float x = proj_at<MODE == 1>(a.x, t, h * a.xs + a.rx + c);
                float y = proj_at<MODE == 1>(a.x, t, h * a.xs + a.rx + half + c);
                x = (float)(T)x;
                y = (float)(T)y;
                const float2 cs = a.cs[(size_t)a.positions[t] * half + c];
                T* o = out + (size_t)t * a.ldo + h * a.os + a.ro;
                o[c] = (T)(x * cs.x - y * cs.y);
                o[half + c] = (T)(y * cs.x + x * cs.y);
            }
            const int pad = a.rot8 - a.rot;
            for (int i = tid; i < nr * pad; i += 256)
                out[(size_t)(r0 + i / pad) * a.ldo + h * a.os + a.ro + a.rot + i % pad] = (T)0.f;
        }
        return;
    }
    const int ldx = a.K + 8;
    if constexpr (MODE == 2) {
        __shared__ float sw[HM_ROWS][256];  // weights of the splits, the common denominator divided out
        __shared__ int s_n[HM_ROWS];        // splits in use: the leading ones
        __shared__ __attribute__((aligned(16))) float4 part[HM_THREADS];
        const int wv = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
        // this wave's weights, a quarter of the depth of 32 columns, are on their way while the sums are merged
        const bf16* w = reinterpret_cast<const bf16*>(a.w) + (size_t)h * a.N * a.K + 8 * g;
        const int n0 = blockIdx.x * HP_COLS + 32 * (wv & 3), kq = 32 * (wv >> 2);
        u32x4 wf[HM_DEPTH][2];
#pragma unroll
        for (int j = 0; j < HM_DEPTH; ++j)
#pragma unroll
            for (int q = 0; q < 2; ++q)
                wf[j][q] = *reinterpret_cast<const u32x4*>(w + (size_t)min(n0 + 16 * q + r16, a.N - 1) * a.K +
                                                           min(kq + 128 * j, a.K - 32));
        if (wv < nr) {
            const float2* m = reinterpret_cast<const float2*>(a.ml) + ((size_t)(r0 + wv) * a.H + h) * a.splits;
            float mx[4], sm[4], best = -INFINITY;
            int n = 0;
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int sp = lane + 64 * q;
                const float2 v = sp < a.splits ? m[sp] : make_float2(-INFINITY, 0.f);
                mx[q] = v.x;
                sm[q] = v.y;
                best = fmaxf(best, v.x);
                n += __popcll(__ballot(v.x != -INFINITY));
            }
            best = wave_max(best);
            float den = 0.f;
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                mx[q] = mx[q] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mx[q] - best);
                den += mx[q] * sm[q];
            }
            den = wave_sum(den);
#pragma unroll
            for (int q = 0; q < 4; ++q) sw[wv][lane + 64 * q] = mx[q] / den;
            if (lane == 0) s_n[wv] = n;
        }
        __syncthreads();
        // thread = (share of the splits, row, four columns)
        const int v4 = a.xk / 4, items = nr * v4, shares = HM_THREADS / items;
        const int sh = tid / items, r = tid % items / v4, k = 4 * (tid % v4);
        if (sh < shares) {
            float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
            const float* p = a.po + ((size_t)(r0 + r) * a.H + h) * a.splits * a.xk + k;
            const int ns = s_n[r];
#pragma unroll 8
            for (int sp = sh; sp < ns; sp += shares) {
                const float4 v = *reinterpret_cast<const float4*>(p + (size_t)sp * a.xk);
                const float f = sw[r][sp];
                acc.x += f * v.x; acc.y += f * v.y; acc.z += f * v.z; acc.w += f * v.w;
            }
            part[tid] = acc;
        }
        __syncthreads();
        for (int i = tid; i < HP_ROWS * (a.K / 4); i += HM_THREADS) {
            const int row = i / (a.K / 4), c = i % (a.K / 4);
            float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
            if (row < nr && c < v4)
                for (int q = 0; q < shares; ++q) {
                    const float4 v = part[q * items + row * v4 + c];
                    acc.x += v.x; acc.y += v.y; acc.z += v.z; acc.w += v.w;
                }
            store4(sx + row * ldx + 4 * c, acc);
        }
        __syncthreads();
        f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int j = 0; j < HM_DEPTH; ++j)
            if (kq + 128 * j < a.K) {
                const bf16x8 xf = *reinterpret_cast<const bf16x8*>(sx + r16 * ldx + 8 * g + kq + 128 * j);
#pragma unroll
                for (int q = 0; q < 2; ++q)
                    acc[q] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf[j][q]), xf, acc[q], 0, 0, 0);
            }
        // the four quarters of the depth: rows of four lanes each
        f32x4* quarter = reinterpret_cast<f32x4*>(part);
        if (r16 < HM_ROWS)
#pragma unroll
            for (int q = 0; q < 2; ++q) quarter[(wv * 2 + q) * 16 + 4 * g + r16] = acc[q];
        __syncthreads();
        if (tid < 128 * HM_ROWS / 4) {  // thread = (16-column group, lane group, row)
            const int c16 = tid >> 4, gg = (tid >> 2) & 3, row = tid & 3;
            const int n = blockIdx.x * HP_COLS + 16 * c16 + 4 * gg;  // N % 8 == 0
            f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < 4; ++kk) y += quarter[((4 * kk + (c16 >> 1)) * 2 + (c16 & 1)) * 16 + 4 * gg + row];
            if (row < nr && n < a.N)
                store4(reinterpret_cast<T*>(a.out) + (size_t)(r0 + row) * a.ldo + h * a.os + n,
                       make_float4(y[0], y[1], y[2], y[3]));
        }
        return;
    } else {
        const int v8 = a.K / 8;
        for (int i = tid; i < HP_ROWS * v8; i += 256) {
            const int r = i / v8, k = 8 * (i % v8);
            float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (r < nr && k < a.xk) proj8<MODE == 1>(a.x, r0 + r, h * a.xs + k, f);
            store8(sx + r * ldx + k, f);
        }
    }
    __syncthreads();
    T* out = reinterpret_cast<T*>(a.out);
    if constexpr (sizeof(T) == 2) {
        const int wv = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
        const bf16* w = reinterpret_cast<const bf16*>(a.w) + (size_t)h * a.N * a.K;
        const int n0 = blockIdx.x * HP_COLS + 32 * wv;
        f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        const bf16* w0 = w + (size_t)min(n0 + r16, a.N - 1) * a.K + 8 * g;
        const bf16* w1 = w + (size_t)min(n0 + 16 + r16, a.N - 1) * a.K + 8 * g;
        const bf16* xr = reinterpret_cast<const bf16*>(sx) + r16 * ldx + 8 * g;
#pragma unroll 4
        for (int k = 0; k < a.K; k += 32) {
            const bf16x8 xf = *reinterpret_cast<const bf16x8*>(xr + k);
            acc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(w0 + k), xf, acc[0], 0, 0, 0);
            acc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(w1 + k), xf, acc[1], 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const int n = n0 + 16 * i + 4 * g;  // N % 8 == 0
            if (r16 < nr && n < a.N)
                store4(out + (size_t)(r0 + r16) * a.ldo + h * a.os + n,
                       make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]));
        }
    } else {
        const float* w = reinterpret_cast<const float*>(a.w) + (size_t)h * a.N * a.K;
        const int rg = tid >> 6;  // rows 4 rg .. + 4
        for (int nn = 0; nn < HP_COLS; nn += 64) {
            const int n = blockIdx.x * HP_COLS + nn + (tid & 63);
            if (n >= a.N) break;
            float acc[4] = {0.f, 0.f, 0.f, 0.f};
            for (int k = 0; k < a.K; k += 4) {
                const float4 wk = *reinterpret_cast<const float4*>(w + (size_t)n * a.K + k);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float4 xk = *reinterpret_cast<const float4*>(sx + (4 * rg + r) * ldx + k);
                    acc[r] += wk.x * xk.x + wk.y * xk.y + wk.z * xk.z + wk.w * xk.w;
                }
            }
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (4 * rg + r < nr) out[(size_t)(r0 + 4 * rg + r) * a.ldo + h * a.os + n] = (T)acc[r];
        }
    }
}

// x: S = 0 bf16 rows, S >= 1 fp32 slabs [S][xrows][ldx], S = -1: split-K partials (po, ml, splits).  w [H][N][K] of the
// output's type; rows = leading rows used.  rot > 0: the rotated tail (HeadArgs).
MRSUM_API int mrsum_head_product(const void* x, int S, int ldx, int xrows, int rows, int xs, int xk, const void* w, int N,
                                 int K, void* out, int f32, int os, int ldo, int H, int rot, int rot8, int rx, int ro,
                                 const void* cs, const int* positions, const float* po, const float* ml, int splits,
                                 hipStream_t s) {
    if (rows <= 0) return 0;
    if (N <= 0 || N % 8 || K % 32 || xk % 8 || xk > K || os % 4 || ldo % 4 || H <= 0 || H > 65535 || rot % 2 ||
        ceil_div(rows, S < 0 ? 1 : HP_ROWS) > 65535 ||
        (S < 0 && (f32 || rot || !po || !ml || splits < 1 || splits > 256 || HM_ROWS * (xk / 4) > HM_THREADS || K > 128 * HM_DEPTH)) ||
        (S >= 0 && (rows > xrows || ldx % 8 || xs % 8)) || (f32 && S < 1))
        return (int)hipErrorInvalidValue;
    // as few rows a block as fill the CUs
    const int mrows = std::max(1, std::min(HM_ROWS, rows * H / 256));
    const HeadArgs a{ProjSrc{x, S, (size_t)xrows * ldx, ldx}, xs, xk, w, N, K, out, os, ldo, rows, H, rot, rot8, rx, ro,
                     (const float2*)cs, positions, po, ml, splits, mrows};
    const int rb = S < 0 ? mrows : HP_ROWS;
    const dim3 g(ceil_div(N, HP_COLS) + (rot ? 1 : 0), H, ceil_div(rows, rb));
    const size_t lds = (size_t)HP_ROWS * (K + 8) * (f32 ? 4 : 2);
    if (lds > 40 * 1024) return (int)hipErrorInvalidValue;
    if (f32) head_product_kernel<float, 1><<<g, 256, lds, s>>>(a);
    else if (S < 0) head_product_kernel<bf16, 2><<<g, HM_THREADS, lds, s>>>(a);
    else if (S) head_product_kernel<bf16, 1><<<g, 256, lds, s>>>(a);
    else head_product_kernel<bf16, 0><<<g, 256, lds, s>>>(a);
    return (int)hipGetLastError();
}

// ------------------------------------------------------------------------------------------------ query rotation
// 16-bit rows: the rotated parts in place (out = the rows).  Slabs: whole rows summed, turned and written.
template <bool PARTS>
__global__ __launch_bounds__(256) void latent_rope_kernel(ProjSrc src, int first, bf16* __restrict__ out, int ldo, int H,
                                                          int qw, int rx, int rot, const float2* __restrict__ cs,
                                                          const int* __restrict__ positions) {
    const int t = blockIdx.x, half = rot / 2;
    const float2* c = cs + (size_t)positions[first + t] * half;
    bf16* o = out + (size_t)t * ldo;
    if constexpr (PARTS) {
        for (int p = threadIdx.x; p < H * qw / 8; p += 256) {
            const int col = 8 * p, in = col % qw;
            float v[8];
            proj8<true>(src, first + t, col, v);
            if (in >= rx) {
                const int base = col - in + rx;
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int d = in - rx + j;
                    if (d >= rot) continue;
                    const int i = d < half ? d : d - half;
                    const float y = (float)(bf16)proj_at<true>(src, first + t, base + (d < half ? d + half : i));
                    const float x = (float)(bf16)v[j];
                    v[j] = d < half ? x * c[i].x - y * c[i].y : x * c[i].x + y * c[i].y;
                }
            }
            store8(o + col, v);
        }
    } else if (half % 8 == 0) {
        const int hp = half / 8;
        for (int p = threadIdx.x; p < H * hp; p += 256) {
            bf16* a = o + (p / hp) * qw + rx + 8 * (p % hp);
            const float2* k = c + 8 * (p % hp);
            float x[8], y[8];
            ld8(a, x);
            ld8(a + half, y);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float u = x[j] * k[j].x - y[j] * k[j].y;
                y[j] = y[j] * k[j].x + x[j] * k[j].y;
                x[j] = u;
            }
            store8(a, x);
            store8(a + half, y);
        }
    } else {
        for (int p = threadIdx.x; p < H * half; p += 256) {
            const int i = p % half;
            bf16* a = o + (p / half) * qw + rx + i;
            const float x = (float)a[0], y = (float)a[half];
            a[0] = (bf16)(x * c[i].x - y * c[i].y);
            a[half] = (bf16)(y * c[i].x + x * c[i].y);
        }
    }
}

// rows [first, T) of q (S = 0: bf16 rows [T][ld], turned in place; S >= 1: fp32 slabs -> out [T - first][ldo])
MRSUM_API int mrsum_latent_rope(void* q, int S, int ld, int T, int first, void* out, int ldo, int H, int qw, int rx, int rot,
                                const void* cs, const int* positions, hipStream_t s) {
    if (T <= first) return 0;
    if (first < 0 || qw % 8 || rx % 8 || rot % 2 || rx + rot > qw || H * qw > ld || ld % 8 || (S && (ldo < H * qw || ldo % 8)))
        return (int)hipErrorInvalidValue;
    if (S) {
        latent_rope_kernel<true><<<T - first, 256, 0, s>>>(ProjSrc{q, S, (size_t)T * ld, ld}, first, (bf16*)out, ldo, H, qw,
                                                           rx, rot, (const float2*)cs, positions);
    } else {
        latent_rope_kernel<false><<<T - first, 256, 0, s>>>(ProjSrc{q, 0, 0, ld}, first, (bf16*)q + (size_t)first * ld, ld, H,
                                                            qw, rx, rot, (const float2*)cs, positions);
    }
    return (int)hipGetLastError();
}

// ------------------------------------------------------------------------------------------------ gathering
// pages: (block-table row, page of the sequence, first destination row, rows) per block
__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16* __restrict__ cache, const int4* __restrict__ pages,
                                                            const int* __restrict__ bt, int bt_stride, int row, int width,
                                                            bf16* __restrict__ out) {
    const int4 e = pages[blockIdx.x];
    const uint4* src = reinterpret_cast<const uint4*>(cache + (size_t)bt[(size_t)e.x * bt_stride + e.y] * 64 * row);
    uint4* dst = reinterpret_cast<uint4*>(out + (size_t)e.z * width);
    const int rv = row / 8, wv = width / 8;
    for (int i = threadIdx.x; i < e.w * wv; i += 256) {
        const int r = i / wv, c = i % wv;
        dst[i] = c < rv ? src[r * rv + c] : make_uint4(0, 0, 0, 0);
    }
}

MRSUM_API int mrsum_latent_gather(const void* cache, const void* pages, int n_pages, const int* bt, int bt_stride, int row,
                                  int width, void* out, hipStream_t s) {
    if (n_pages <= 0) return 0;
    if (row % 8 || width % 8 || width < row) return (int)hipErrorInvalidValue;
    latent_gather_kernel<<<n_pages, 256, 0, s>>>((const bf16*)cache, (const int4*)pages, bt, bt_stride, row, width,
                                                 (bf16*)out);
    return (int)hipGetLastError();
}
