// Attention kernels of latent attention (latent.hip prepares their operands).
//
// latent_prefill: causal flash attention of prompt portions over keys and values expanded from the latents.  A workgroup
// runs 256 query rows of one head, 32 per wave, against 64-key tiles in a two-stage LDS ring: a key row is [expanded
// unrotated part of the head | rotated part shared by the heads], values come from the expansion.  The products are the
// swapped ones of attn_prefill.hip (S^T = K Q^T, O^T = V^T P^T on v_mfma_f32_32x32x16_bf16), the softmax weights enter as
// two bf16 terms.  Row strides are padded so that 16-lane groups of either kind of LDS read hit distinct banks.
//
// latent_decode: split-K attention of single tokens with absorbed queries over the cached rows themselves (one row per
// token for all heads; its first columns are also the value).  A workgroup runs up to 32 heads of one sequence over its
// share of pages: a page's rows sit in LDS (the next page's in registers), every wave scores and exponentiates a 16-key x
// 16-head tile, and after the weights have crossed LDS every wave sums its own block of value columns.  Output: unmerged
// partial sums.
#include "common.h"

namespace {
typedef short s4 __attribute__((ext_vector_type(4)));
typedef short s8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) s4 lds_s4;

__device__ __forceinline__ bf16x8 as8(u32x4 v) { return __builtin_bit_cast(bf16x8, v); }
__device__ __forceinline__ bf16x8 tr8(const bf16* lo, const bf16* hi) {
    const s4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)lo);
    const s4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)hi);
    return __builtin_bit_cast(bf16x8, (s8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]}));
}
// maximum over the four 16-lane groups
__device__ __forceinline__ float groups_max(float v) {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
    const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float halves(float v, bool max) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    const float a = __uint_as_float(r[0]), b = __uint_as_float(r[1]);
    return max ? fmaxf(a, b) : a + b;
}

constexpr int BN = 64, NTHR = 512;
constexpr float RESCALE_LOG2 = 8.0f;  // the running maximum moves when a row's maximum grew by more than this

struct LatPrefill {
    const bf16* q;       // [T][ldq], head h at columns [h * qw, + qw)
    int ldq, qw;
    const bf16* kv;      // expanded rows: head h's key at h * dim8, its value at v_at + h * vp
    int ldkv, dim8, v_at, vp;
    const bf16* lat;     // gathered rows: rotated part at rot_at
    int ldl, rot_at;
    const int* cu;       // [portions + 1] query rows
    const int* prefix;   // [portions] positions before the portion
    const int* base;     // [portions + 1] first key row
    const int2* items;   // (portion, first query row), heaviest first
    int n_items, H;
    bf16* out;
    int ldo;
    float scale_log2;
    int head_major;
};
}  // namespace

template <int KC, int VC>
__global__ __launch_bounds__(NTHR, 1) void latent_prefill_kernel(const LatPrefill a) {
    constexpr int LK = 16 * KC + 8, LV = 32 * (VC | 1);  // row strides
    constexpr int KIT = KC / 4, VIT = VC / 2;            // 16-byte pieces a thread stages: row tid / 8, piece tid % 8 + 8 i
    constexpr int STAGE = BN * (LK + LV);
    __shared__ __attribute__((aligned(16))) bf16 lds[2 * STAGE];
    const int item = a.head_major ? blockIdx.x % a.n_items : blockIdx.x / a.H;
    const int h = a.head_major ? blockIdx.x / a.n_items : blockIdx.x % a.H;
    const int2 it = a.items[item];
    const int seq = it.x, tid = threadIdx.x, lane = tid & 63, half = lane >> 5, r32 = lane & 31, w = tid >> 6;
    const int s0 = a.cu[seq], len = a.cu[seq + 1] - s0, pre = a.prefix[seq], k0 = a.base[seq];
    const int q0 = it.y + 32 * w, qi = q0 + r32;
    bf16x8 qf[KC];
    {
        const bool ok = qi < len;
        const bf16* qp = a.q + (size_t)(s0 + (ok ? qi : 0)) * a.ldq + h * a.qw;
#pragma unroll
        for (int ks = 0; ks < KC; ++ks) {
            const int c = 16 * ks + 8 * half;
            u32x4 v = *reinterpret_cast<const u32x4*>(qp + min(c, a.qw - 8));
            if (!ok || c >= a.qw) v = u32x4{0, 0, 0, 0};
            qf[ks] = as8(v);
        }
    }
    const int kend = pre + min(len, it.y + 256), ntiles = (kend + BN - 1) / BN, klast = pre + len - 1;
    // Staging reads are unconditional: rows past the sequence repeat its last one (masked), columns past the key's or
    // value's width repeat a valid piece (the query is zero there, such outputs are not stored).
    const int srow = tid >> 3, sp = tid & 7;
    u32x4 kreg[KIT], vreg[VIT];
#define LOAD_TILE(t)                                                                                     \
    {                                                                                                    \
        const int key_ = k0 + min((t) * BN + srow, klast);                                               \
        const bf16* kr_ = a.kv + (size_t)key_ * a.ldkv;                                                  \
        const bf16* lr_ = a.lat + (size_t)key_ * a.ldl + a.rot_at;                                       \
        _Pragma("unroll") for (int i = 0; i < KIT; ++i) {                                                \
            const int c_ = min(8 * (sp + 8 * i), a.qw - 8);                                              \
            const bf16* p_ = c_ < a.dim8 ? kr_ + h * a.dim8 + c_ : lr_ + (c_ - a.dim8);                  \
            kreg[i] = *reinterpret_cast<const u32x4*>(p_);                                               \
        }                                                                                                \
        _Pragma("unroll") for (int i = 0; i < VIT; ++i)                                                  \
            vreg[i] = *reinterpret_cast<const u32x4*>(kr_ + a.v_at + h * a.vp + min(8 * (sp + 8 * i), a.vp - 8)); \
    }
#define STORE_TILE(st)                                                                                   \
    {                                                                                                    \
        _Pragma("unroll") for (int i = 0; i < KIT; ++i)                                                  \
            *reinterpret_cast<u32x4*>(lds + (st) + srow * LK + 8 * (sp + 8 * i)) = kreg[i];              \
        _Pragma("unroll") for (int i = 0; i < VIT; ++i)                                                  \
            *reinterpret_cast<u32x4*>(lds + (st) + BN * LK + srow * LV + 8 * (sp + 8 * i)) = vreg[i];    \
    }
    f32x16 o[VC];
#pragma unroll
    for (int dt = 0; dt < VC; ++dt) o[dt] = f32x16{};
    float m = -INFINITY, l = 0.f;
    LOAD_TILE(0)
    STORE_TILE(0)
    LOAD_TILE(min(1, ntiles - 1))
    const int wave_last = pre + q0 + 31;  // absolute position of the wave's last row
    const int g = lane >> 4, q4 = (lane & 15) >> 2, p4 = lane & 3;
    for (int t = 0; t < ntiles; ++t) {
        const int cur = (t & 1) * STAGE, kv0 = t * BN;
        __syncthreads();  // tile t visible; every wave is done with tile t - 1
        STORE_TILE(STAGE - cur)
        LOAD_TILE(min(t + 2, ntiles - 1))
        if (kv0 > wave_last) continue;  // wave-uniform: tiles wholly above the diagonal
        const bf16* sk = lds + cur;
        const bf16* sv = sk + BN * LK;
        f32x16 sacc[2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            u32x4 kf[KC];
#pragma unroll
            for (int ks = 0; ks < KC; ++ks)
                kf[ks] = *reinterpret_cast<const u32x4*>(sk + (32 * kt + r32) * LK + 16 * ks + 8 * half);
            sacc[kt] = f32x16{};
#pragma unroll
            for (int ks = 0; ks < KC; ++ks)
                sacc[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(as8(kf[ks]), qf[ks], sacc[kt], 0, 0, 0);
        }
        // reads run ahead of the products
        __builtin_amdgcn_sched_group_barrier(0x100, 6, 0);
#pragma unroll
        for (int i = 0; i < 2 * KC - 6; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
            __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
        __builtin_amdgcn_sched_group_barrier(0x008, 6, 0);
        // key of register i: 32 kt + (i & 3) + 8 (i >> 2) + 4 half
        const int kmax = pre + min(qi, len - 1) - kv0 - 4 * half;
        if (kv0 + BN - 1 > pre + q0 || kv0 + BN > pre + len) {
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int i = 0; i < 16; ++i)
                    sacc[kt][i] = 32 * kt + (i & 3) + 8 * (i >> 2) <= kmax ? sacc[kt][i] : -INFINITY;
        }
        float mt = -INFINITY;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
            for (int i = 0; i < 16; ++i) mt = fmaxf(mt, sacc[kt][i]);
        const float mc = halves(mt, true) * a.scale_log2;
        if (__ballot(mc > m + RESCALE_LOG2)) {  // key 0 is visible to every row, so m is finite after tile 0
            const float mn = fmaxf(m, mc), alpha = __builtin_amdgcn_exp2f(m - mn);
            m = mn;
            l *= alpha;
#pragma unroll
            for (int dt = 0; dt < VC; ++dt) o[dt] *= alpha;
        }
        float ls = 0.f;
        bf16x8 pf[2][2], pl[2][2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const float p = __builtin_amdgcn_exp2f(fmaf(sacc[kt][i], a.scale_log2, -m));
                ls += p;
                pf[kt][i >> 3][i & 7] = (bf16)p;
                pl[kt][i >> 3][i & 7] = (bf16)(p - (float)(bf16)p);
            }
        l += ls;
#pragma unroll
        for (int dt = 0; dt < VC; ++dt) {
            bf16x8 va[2][2];
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int s = 0; s < 2; ++s) {
                    const bf16* vr = sv + (32 * kt + 16 * s + 4 * (g >> 1) + q4) * LV + 32 * dt + 16 * (g & 1) + 4 * p4;
                    va[kt][s] = tr8(vr, vr + 8 * LV);
                }
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
#pragma unroll
                for (int s = 0; s < 2; ++s) {
                    o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va[kt][s], pf[kt][s], o[dt], 0, 0, 0);
                    o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va[kt][s], pl[kt][s], o[dt], 0, 0, 0);
                }
        }
        __builtin_amdgcn_sched_group_barrier(0x100, 8, 1);
#pragma unroll
        for (int i = 0; i < 4 * VC - 4; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, 2, 1);
            __builtin_amdgcn_sched_group_barrier(0x100, 2, 1);
        }
        __builtin_amdgcn_sched_group_barrier(0x008, 8, 1);
    }
#undef LOAD_TILE
#undef STORE_TILE
    // register i of block dt: value column 32 dt + (i & 3) + 8 (i >> 2) + 4 half; halves trade so that a lane stores 16 bytes
    const float inv = 1.f / halves(l, false);
    bf16* op = a.out + (size_t)(s0 + qi) * a.ldo + h * a.vp + 8 * half;
#pragma unroll
    for (int dt = 0; dt < VC; ++dt)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const uint32_t a0 = pack2(o[dt][8 * j + 0] * inv, o[dt][8 * j + 1] * inv);
            const uint32_t a1 = pack2(o[dt][8 * j + 2] * inv, o[dt][8 * j + 3] * inv);
            const uint32_t b0 = pack2(o[dt][8 * j + 4] * inv, o[dt][8 * j + 5] * inv);
            const uint32_t b1 = pack2(o[dt][8 * j + 6] * inv, o[dt][8 * j + 7] * inv);
            const auto r0 = __builtin_amdgcn_permlane32_swap(a0, b0, false, false);
            const auto r1 = __builtin_amdgcn_permlane32_swap(a1, b1, false, false);
            if (qi < len && 32 * dt + 16 * j + 8 * half < a.vp)
                *reinterpret_cast<uint4*>(op + 32 * dt + 16 * j) = make_uint4(r0[0], r1[0], r0[1], r1[1]);
        }
}

// q rows [Tq][ldq] of prompt portions, heads of qw = dim8 + rotated columns; key rows as in LatPrefill; items: (portion,
// first query row) in blocks of 256 rows.  out: head h of a row at columns [h * vp, (h + 1) * vp).  form: 16-column key
// steps of the instantiation (4, 8, 12: qw <= 64, 128, 192; vp <= 64, 128, 128).
MRSUM_API int mrsum_latent_prefill(const void* q, int ldq, int qw, const void* kv, int ldkv, int dim8, int v_at, int vp,
                                   const void* lat, int ldl, int rot_at, const int* cu, const int* prefix, const int* base,
                                   const void* items, int n_items, int H, void* out, int ldo, float scale, int form,
                                   hipStream_t s) {
    if (n_items <= 0) return 0;
    const int vmax = form == 4 ? 64 : 128;
    if ((form != 4 && form != 8 && form != 12) || qw > 16 * form || qw < 8 || vp > vmax || vp < 8 || qw % 8 || vp % 8 ||
        dim8 % 8 || dim8 > qw || ldq % 8 || ldkv % 8 || ldl % 8 || rot_at % 8 || v_at % 8 || ldo % 8 || H <= 0 ||
        ldq < H * qw || ldkv < v_at + H * vp || v_at < H * dim8 || ldl < rot_at + qw - dim8 || ldo < H * vp ||
        (long long)n_items * H > 0x7fffffff)
        return (int)hipErrorInvalidValue;
    const int blocks = n_items * H;
    const LatPrefill a{(const bf16*)q, ldq, qw, (const bf16*)kv, ldkv, dim8, v_at, vp, (const bf16*)lat, ldl, rot_at, cu,
                       prefix, base, (const int2*)items, n_items, H, (bf16*)out, ldo, scale * 1.4426950408889634f,
                       blocks > 8 * 256};
    if (form == 4) latent_prefill_kernel<4, 2><<<blocks, NTHR, 0, s>>>(a);
    else if (form == 8) latent_prefill_kernel<8, 4><<<blocks, NTHR, 0, s>>>(a);
    else latent_prefill_kernel<12, 4><<<blocks, NTHR, 0, s>>>(a);
    return (int)hipGetLastError();
}

// ------------------------------------------------------------------------------------------------ decoded tokens
namespace {
constexpr int DH = 32;  // heads per workgroup

struct LatDecode {
    const bf16* q;      // [B][H * row] absorbed queries
    const bf16* cache;  // [pages][64][row]
    const int* bt;
    int bt_stride;
    const int* positions;
    int H, rank, row, S;
    float scale_log2;
    float* po;          // [B][H][S][rank]
    float2* ml;         // [B][H][S] (maximum in log2 units, sum)
};
}  // namespace

// KB: 32-column blocks of a cached row, VB: 128-column blocks of the latent.  Grid (S, ceil(H / 32), B).  Two barriers a
// page: the next page's registers go to the other LDS stage between them, when every wave is past the page before.
template <int KB, int VB>
__global__ __launch_bounds__(512, 1) void latent_decode_kernel(const LatDecode a) {
    constexpr int LK = 32 * KB + 8, LP = BN + 8, IT = KB / 2;
    __shared__ __attribute__((aligned(16))) bf16 sk[2][BN * LK];
    __shared__ __attribute__((aligned(16))) bf16 sph[DH * LP];  // softmax weights, hi and lo terms
    __shared__ __attribute__((aligned(16))) bf16 spl[DH * LP];
    __shared__ __attribute__((aligned(16))) float smax[DH][4];  // maxima of the four 16-key blocks
    const int sp = blockIdx.x, h0 = DH * blockIdx.y, b = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, r16 = lane & 15, g = lane >> 4, q4 = r16 >> 2, p4 = 4 * (r16 & 3);
    const int w = __builtin_amdgcn_readfirstlane(tid >> 6), kb4 = w & 3, hb = w >> 2;
    bf16x8 qf[KB];  // this wave's 16 heads
    {
        const int h = h0 + 16 * hb + r16;
        const bf16* qp = a.q + ((size_t)b * a.H + min(h, a.H - 1)) * a.row;
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
            const int c = 32 * kb + 8 * g;
            u32x4 v = *reinterpret_cast<const u32x4*>(qp + min(c, a.row - 8));
            if (c >= a.row || h >= a.H) v = u32x4{0, 0, 0, 0};
            qf[kb] = as8(v);
        }
    }
    const int pos = a.positions[b], pages = pos / BN + 1;
    const int used = min(a.S, pages);  // splits past them are empty
    const int p0 = sp < used ? (int)((long long)pages * sp / used) : 0;
    const int p1 = sp < used ? (int)((long long)pages * (sp + 1) / used) : 0;
    const int* bt = a.bt + (size_t)b * a.bt_stride;
    const int rc = a.row / 8, total = BN * rc;  // 16-byte pieces of a row / of a page
    u32x4 reg[IT];
    int at[IT];  // LDS offset of piece tid + 512 i (past the page: the last piece once more)
#pragma unroll
    for (int i = 0; i < IT; ++i) {
        const int c = min(tid + 512 * i, total - 1);
        at[i] = c / rc * LK + 8 * (c % rc);
    }
    // the id of the page after the one being fetched is read ahead, so that fetching never waits for it
    int id = 0;
#define LOAD_PAGE(p)                                                                                    \
    {                                                                                                   \
        const bf16* pg_ = a.cache + (size_t)id * BN * a.row;                                            \
        id = bt[min((p) + 1, p1 - 1)];                                                                  \
        _Pragma("unroll") for (int i = 0; i < IT; ++i)                                                  \
            reg[i] = *reinterpret_cast<const u32x4*>(pg_ + 8 * min(tid + 512 * i, total - 1));          \
    }
    f32x4 acc[VB][2];
    float m[2] = {-INFINITY, -INFINITY}, l = 0.f;  // maxima of heads r16, 16 + r16; this lane's share of head 16 hb + r16's sum
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) acc[vb][0] = acc[vb][1] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (p0 < p1) {
        id = bt[p0];
        LOAD_PAGE(p0)
        // columns past the row: zeros in both stages
        const int rz = 4 * KB - rc;
        for (int i = tid; i < 2 * BN * rz; i += 512)
            *reinterpret_cast<u32x4*>(&sk[0][0] + (i / rz) * LK + 8 * (rc + i % rz)) = u32x4{0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < IT; ++i) *reinterpret_cast<u32x4*>(&sk[0][0] + at[i]) = reg[i];
        LOAD_PAGE(min(p0 + 1, p1 - 1))
        __syncthreads();
        for (int p = p0; p < p1; ++p) {
            const bf16* cur = &sk[(p - p0) & 1][0];
            f32x4 s;
            {
                f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
                const bf16* kr = cur + (16 * kb4 + r16) * LK + 8 * g;
#pragma unroll
                for (int kb = 0; kb < KB; kb += 2) {
                    s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(kr + 32 * kb), qf[kb], s0,
                                                                 0, 0, 0);
                    s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(kr + 32 * kb + 32),
                                                                 qf[kb + 1], s1, 0, 0, 0);
                }
                s = s0 + s1;
            }
            const int kmax = pos - BN * p - 16 * kb4 - 4 * g;  // last visible of this lane's four keys
            float mx = -INFINITY;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                s[j] = j <= kmax ? s[j] * a.scale_log2 : -INFINITY;
                mx = fmaxf(mx, s[j]);
            }
            mx = groups_max(mx);
            if (g == 0) smax[16 * hb + r16][kb4] = mx;
            __syncthreads();
            float alpha[2];
#pragma unroll
            for (int hh = 0; hh < 2; ++hh) {
                const f32x4 v = *reinterpret_cast<const f32x4*>(&smax[16 * hh + r16][0]);
                const float mn = fmaxf(m[hh], fmaxf(fmaxf(v[0], v[1]), fmaxf(v[2], v[3])));  // key 0 of a page is visible
                alpha[hh] = __builtin_amdgcn_exp2f(m[hh] - mn);
                m[hh] = mn;
            }
            {
                const float mh = hb ? m[1] : m[0];
                float e[4], lo[4];
#pragma unroll
                for (int j = 0; j < 4; ++j) e[j] = __builtin_amdgcn_exp2f(s[j] - mh);
                l = l * (hb ? alpha[1] : alpha[0]) + (e[0] + e[1]) + (e[2] + e[3]);
#pragma unroll
                for (int j = 0; j < 4; ++j) lo[j] = e[j] - (float)(bf16)e[j];
                const int o = (16 * hb + r16) * LP + 16 * kb4 + 4 * g;
                *reinterpret_cast<uint2*>(sph + o) = make_uint2(pack2(e[0], e[1]), pack2(e[2], e[3]));
                *reinterpret_cast<uint2*>(spl + o) = make_uint2(pack2(lo[0], lo[1]), pack2(lo[2], lo[3]));
            }
            if (p + 1 < p1) {
                bf16* nxt = &sk[(p - p0 + 1) & 1][0];
#pragma unroll
                for (int i = 0; i < IT; ++i) *reinterpret_cast<u32x4*>(nxt + at[i]) = reg[i];
                LOAD_PAGE(min(p + 2, p1 - 1))
            }
#pragma unroll
            for (int vb = 0; vb < VB; ++vb) {
                acc[vb][0] *= alpha[0];
                acc[vb][1] *= alpha[1];
            }
            __syncthreads();
            bf16x8 ph[2][2], pl[2][2];
#pragma unroll
            for (int hh = 0; hh < 2; ++hh)
#pragma unroll
                for (int kk = 0; kk < 2; ++kk) {
                    const int o = (16 * hh + r16) * LP + 32 * kk + 8 * g;
                    ph[hh][kk] = *reinterpret_cast<const bf16x8*>(sph + o);
                    pl[hh][kk] = *reinterpret_cast<const bf16x8*>(spl + o);
                }
#pragma unroll
            for (int vb = 0; vb < VB; ++vb) {
                const int r0 = 16 * (w + 8 * vb);
                if (r0 < a.rank) {
#pragma unroll
                    for (int kk = 0; kk < 2; ++kk) {
                        const bf16* vr = cur + (32 * kk + 8 * g + q4) * LK + r0 + p4;
                        const bf16x8 vt = tr8(vr, vr + 4 * LK);
#pragma unroll
                        for (int hh = 0; hh < 2; ++hh) {
                            acc[vb][hh] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, ph[hh][kk], acc[vb][hh], 0, 0, 0);
                            acc[vb][hh] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pl[hh][kk], acc[vb][hh], 0, 0, 0);
                        }
                    }
                }
            }
        }
    }
#undef LOAD_PAGE
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
        const int h = h0 + 16 * hh + r16;
        if (h >= a.H || p0 == p1) continue;
        const size_t e = ((size_t)b * a.H + h) * a.S + sp;
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
            const int r = 16 * (w + 8 * vb) + 4 * g;
            if (r < a.rank) *reinterpret_cast<f32x4*>(a.po + e * a.rank + r) = acc[vb][hh];
        }
    }
    // the sum of a head: lane groups, then the four key blocks (waves of the same half)
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    __syncthreads();
    if (g == 0) smax[16 * hb + r16][kb4] = l;
    __syncthreads();
    if (tid < 2 * 64 && g == 0) {
        const int hh = w, h = h0 + 16 * hh + r16;
        const f32x4 v = *reinterpret_cast<const f32x4*>(&smax[16 * hh + r16][0]);
        if (h < a.H)
            a.ml[((size_t)b * a.H + h) * a.S + sp] = make_float2(hh ? m[1] : m[0], (v[0] + v[1]) + (v[2] + v[3]));
    }
}

// q [B][H * row] bf16; po [B][H][S][rank] fp32, ml [B][H][S] pairs.  rank % 8 == 0, row % 8 == 0; (rank, row) up to
// (128, 128), (256, 320) or (512, 576).
MRSUM_API int mrsum_latent_decode(const void* q, const void* cache, const int* bt, int bt_stride, const int* positions, int B,
                                  int H, int rank, int row, int S, float scale, float* po, float* ml, hipStream_t s) {
    if (B <= 0) return 0;
    if (H <= 0 || S <= 0 || S > 65535 || B > 65535 || rank % 8 || row % 8 || rank <= 0 || rank > row || rank > 512 || row > 576)
        return (int)hipErrorInvalidValue;
    const LatDecode a{(const bf16*)q, (const bf16*)cache, bt, bt_stride, positions, H, rank, row, S,
                      scale * 1.4426950408889634f, po, (float2*)ml};
    const dim3 grid(S, ceil_div(H, DH), B);
    if (rank <= 128 && row <= 128) latent_decode_kernel<4, 1><<<grid, 512, 0, s>>>(a);
    else if (rank <= 256 && row <= 320) latent_decode_kernel<10, 2><<<grid, 512, 0, s>>>(a);
    else latent_decode_kernel<18, 4><<<grid, 512, 0, s>>>(a);
    return (int)hipGetLastError();
}
